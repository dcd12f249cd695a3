"""Small Gisedra configurations for the tests (none of them anyone's model), edits of their random weights that make a
fault visible, and the comparison of an engine's logits with the plain implementation's, position by position."""
from __future__ import annotations

import os
from typing import Dict

import numpy as np

import plain_gisedra as pg
import replay_util as ru


def rotation(dims, base=5000.0, scaling=None):
    r = {"base": base, "dims": dims}
    if scaling is not None:
        r["scaling"] = scaling
    return r


SCALING = {"factor": 6.0, "low": 1.0, "high": 3.0, "original": 40}


def latent(heads=4, dim=16, rot_dim=8, vdim=24, kv_rank=32, base=5000.0, window=20, scale=None, mlp=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank,
         "scale": scale if scale is not None else (dim + rot_dim) ** -0.5}
    if rot_dim > 0:
        m["rot"] = rotation(rot_dim, base)
    if window is not None:
        m["mask"] = {"size": window}
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def left(heads=4, kv_heads=2, dim=16, vdim=24, conv=3, rot=None, scale=None, window=20, keep_first=3):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv, "scale": scale if scale is not None else dim ** -0.5,
         "rot": rot if rot is not None else rotation(dim // 2, scaling=SCALING)}
    if window is not None:
        m["mask"] = {"size": window, "keep_first": keep_first}
    return m


def right(heads=2, dim=8, vdim=12, decay=None):
    return {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay or [1.0 - 2.0 ** -(3 + 2 * h) for h in range(heads)]}


def pair(a=None, b=None, left_scale=0.7, right_scale=1.1, mlp=None):
    return {"type": "parallel", "mixer": {"left": a or left(), "right": b or right(), "left_scale": left_scale, "right_scale": right_scale},
            "mlp": mlp}


def moe(experts=5, top=2, ff=24):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}


def model(layers, vocab=300, width=64, eps=1e-5, side=8, loop=None):
    c = {"architecture": "Gisedra", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if side is not None:
        c["token_side"] = {"dim": side}
    if loop is not None:
        c["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return c


# single mechanisms: one mixer without a feed-forward, loop or token input, unless that is what is tested
ONLY_LATENT = model([latent()], side=None)
ONLY_LATENT_FULL = model([latent(window=None, heads=3, dim=24, rot_dim=4, vdim=8, kv_rank=20)], width=48, side=None)         # no window
ONLY_LATENT_NO_TURN = model([latent(heads=3, dim=24, rot_dim=0, vdim=8, kv_rank=20)], width=48, side=None)
ONLY_LATENT_NARROW = model([latent(heads=1, dim=32, rot_dim=2, vdim=64, kv_rank=48, window=1, base=30.0)], width=40, side=None)   # sees itself only
ONLY_LATENT_MANY = model([latent(heads=12, dim=8, rot_dim=4, vdim=12, kv_rank=16, window=33)], width=96, side=None)
ONLY_PAIR = model([pair()], side=None)
PAIR_NO_CONV = model([pair(left(conv=0))], side=None)                                               # the left scale without taps to stand in
PAIR_ONE_TAP = model([pair(left(conv=1, heads=2, kv_heads=1), left_scale=1.0, right_scale=1.0)], width=32, side=None)
PAIR_MANY_TAPS = model([pair(left(conv=7, dim=12, vdim=10, heads=3, kv_heads=3, rot=rotation(6, 100.0)))], width=40, side=None)
PAIR_PLAIN_FREQUENCIES = model([pair(left(rot=rotation(16, 300.0)), left_scale=0.5)], side=None)
PAIR_NO_TURN = model([pair(left(rot=rotation(0)), left_scale=1.4)], side=None)
PAIR_NO_WINDOW = model([pair(left(window=None, heads=4, kv_heads=4))], side=None)
PAIR_KEEPS_MORE = model([pair(left(window=4, keep_first=9))], side=None)                            # keeps more than the window holds
PAIR_KEEPS_NONE = model([pair(left(window=12, keep_first=0))], side=None)
PAIR_ONE_HEAD = model([pair(left(heads=1, kv_heads=1, dim=32, vdim=16), right(heads=1, dim=24, vdim=40))], width=48, side=None)
PAIR_TWICE_AS_WIDE = model([pair(left(heads=4, kv_heads=2, dim=32, vdim=64), right(heads=3, dim=40, vdim=16))], side=None)
PAIR_VERY_MANY_HEADS = model([pair(left(heads=64, kv_heads=64, dim=136, vdim=8), right(heads=1, dim=8, vdim=8))], width=32, side=None)   # 70 KB of heads a token
PAIR_UNALIGNED = model([pair(left(heads=3, kv_heads=1, dim=10, vdim=7, rot=rotation(6, scaling=SCALING)), right(heads=3, dim=5, vdim=9))], width=40, side=None)
PAIR_MANY_KEY_COLUMNS = model([pair(left(), right(heads=2, dim=72, vdim=80))], width=48, side=None)
ONLY_EXPERTS = model([latent(mlp=moe())], side=None)
EXPERTS_ALL = model([latent(mlp=moe(experts=3, top=3, ff=16))], width=32, side=None)               # every expert chosen
ONE_EXPERT = model([latent(mlp=moe(experts=1, top=1, ff=32))], width=32, side=None)
TOP_ONE = model([latent(mlp=moe(experts=6, top=1, ff=16))], width=32, side=None)
MANY_EXPERTS = model([latent(mlp=moe(experts=70, top=3, ff=8))], width=32, side=None)              # more than a wavefront has lanes
ONLY_SIDE = model([latent(), latent()], side=8)
SIDE_ONE = model([latent()], width=40, side=1)
SIDE_ODD = model([latent(), latent()], width=44, side=13)
SIDE_WIDE = model([latent()], width=96, side=72)
LOOP_ALL = model([latent(), pair()], side=None, loop=(0, 2, 3))
LOOP_ONE_LAYER = model([latent(), latent(), latent()], side=4, loop=(1, 2, 4))
LOOP_ONCE = model([latent(), pair()], side=None, loop=(1, 2, 1))
# several layers in orders of their own
MIXED_A = model([
    pair(mlp=moe()),
    latent(mlp=moe(experts=7, top=3, ff=16)),
    pair(left(heads=6, kv_heads=2, dim=16, vdim=16, conv=4, window=11, keep_first=5), right(heads=3, dim=16, vdim=8), 1.2, 0.6),
    latent(heads=2, dim=32, rot_dim=16, vdim=32, kv_rank=48, base=900.0, window=37, mlp=moe(experts=4, top=1, ff=32)),
], vocab=257, width=64, eps=1e-6, side=16, loop=(1, 3, 2))
MIXED_B = model([
    latent(heads=6, dim=8, rot_dim=8, vdim=16, kv_rank=24, window=9, mlp=moe(experts=9, top=4, ff=16)),
    latent(heads=3, dim=16, rot_dim=4, vdim=8, kv_rank=56, window=64),
    pair(left(heads=8, kv_heads=8, dim=8, vdim=16, conv=2, window=30, keep_first=1), right(heads=4, dim=12, vdim=24), 0.9, 0.9, mlp=moe(experts=3, top=2, ff=24)),
], vocab=513, width=48, side=12, loop=(0, 2, 2))
# sizes that are multiples of neither 8 nor 4; a width that is odd
ODD = model([
    pair(left(heads=3, kv_heads=1, dim=10, vdim=7, conv=3, rot=rotation(6, scaling=SCALING), window=17, keep_first=2), right(heads=1, dim=5, vdim=9), mlp=moe(experts=5, top=2, ff=13)),
    latent(heads=3, dim=6, rot_dim=2, vdim=9, kv_rank=11, window=23),
    latent(heads=2, dim=7, rot_dim=6, vdim=5, kv_rank=17, window=50, mlp=moe(experts=3, top=2, ff=9)),
], vocab=101, width=43, side=5, loop=(1, 3, 2))
# the sizes of a larger model's layers: the matrix-core kernels
LARGER = model([
    pair(left(heads=4, kv_heads=2, dim=64, vdim=64, conv=4, rot=rotation(32, 10000.0, {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 128}), window=80, keep_first=10),
         right(heads=4, dim=64, vdim=64), mlp=moe(experts=6, top=2, ff=96)),
    latent(heads=4, dim=64, rot_dim=32, vdim=64, kv_rank=128, window=70, mlp=moe(experts=12, top=3, ff=64)),
    pair(left(heads=4, kv_heads=1, dim=64, vdim=128, conv=3, window=100, keep_first=33), right(heads=2, dim=32, vdim=64), mlp=moe(experts=4, top=2, ff=128)),
    latent(heads=8, dim=32, rot_dim=64, vdim=48, kv_rank=224, window=129),
], vocab=211, width=256, side=32, loop=(1, 2, 2))
# scores that single keys dominate: a key that is lost, one too many or turned by the wrong angle changes whole rows
PEAKED = model([pair(left(scale=1.5, window=20, keep_first=3)), latent(scale=1.5, window=26)], width=32, side=None)
PEAKED_TILES = model([pair(left(heads=4, kv_heads=2, dim=32, vdim=32, scale=0.9, window=70, keep_first=6)),
                      latent(heads=4, dim=32, rot_dim=32, vdim=32, kv_rank=64, scale=0.9, window=45)], width=64, side=None)
# memories that hardly decay beside ones that do: what a token far back wrote carries late rows
SLOW = model([pair(left(window=6, keep_first=0), right(heads=3, dim=16, vdim=16, decay=[1.0 - 2.0 ** -11, 0.5, 1.0]), 0.3, 1.5)], width=32, side=None)
# without routed experts (greedy generation in bfloat16: what is generated cannot be chosen to suit a router)
UNROUTED = model([pair(), latent(), pair(left(heads=2, kv_heads=2, dim=32, vdim=32)), latent(heads=2, dim=32, rot_dim=16, vdim=32, kv_rank=48)],
                 vocab=257, side=16, loop=(1, 3, 2))

# name -> tensor name -> (factor, added): the stored tensor times factor plus added
EDITS = {
    # (logits further apart: fewer tokens at which rounding may choose another expert)
    "MIXED_A": {"l0.mlp.router": (3.0, 0.0), "l1.mlp.router": (3.0, 0.0), "l3.mlp.router": (3.0, 0.0)},
    "MIXED_B": {"l0.mlp.router": (3.0, 0.0), "l2.mlp.router": (3.0, 0.0)},
    "ODD": {"l0.mlp.router": (3.0, 0.0), "l2.mlp.router": (3.0, 0.0)},
}


def write_case(name, out_dir, seed=3):
    """The named configuration's folder: random weights, with the case's edits."""
    from mini_llm_amd import write_random_model
    write_random_model(dict(globals()[name]), out_dir, seed)
    if name in EDITS:
        from safetensors.torch import load_file, save_file
        path = os.path.join(out_dir, "model.safetensors")
        t = load_file(path)
        for tensor, (factor, added) in EDITS[name].items():
            t[tensor] = (t[tensor].float() * factor + added).to(t[tensor].dtype).contiguous()
        save_file(t, path)
    return out_dir


# rms(difference, mean taken off) / rms(logits, mean taken off) of a row may be at most this
TOL = {"float32": 2e-5, "bfloat16": 3e-2}
TOL_PEAKED = 1e-4
CLOSE_CALL = 0.015      # a gap between two router logits below which bfloat16 rounding may choose the other expert
CLOSE_REACH = 8         # positions behind such a token that still carry it most

_plain: Dict[tuple, np.ndarray] = {}
_weights: Dict[str, tuple] = {}
_calls: Dict[tuple, np.ndarray] = {}
_moves: Dict[tuple, np.ndarray] = {}
_decisive: Dict[tuple, dict] = {}


def plain_model(model_dir):
    if model_dir not in _weights:
        _weights[model_dir] = pg.read_model(model_dir)
    return _weights[model_dir]


def plain_logits(model_dir, toks) -> np.ndarray:
    key = (model_dir, tuple(toks))
    if key not in _plain:
        cfg, w = plain_model(model_dir)
        _plain[key] = pg.logits(cfg, w, list(toks)).numpy()
    return _plain[key]


def closest_call(model_dir, toks) -> np.ndarray:
    key = (model_dir, tuple(toks))
    if key not in _calls:
        cfg, w = plain_model(model_dir)
        _calls[key] = pg.closest_call(cfg, w, list(toks)).numpy()
    return _calls[key]


def row_error(got, ref) -> float:
    d = got.astype(np.float64) - ref
    d = d - d.mean()
    r = ref - ref.mean()
    return float(np.sqrt((d * d).mean()) / np.sqrt((r * r).mean()))


def moves(model_dir, toks) -> np.ndarray:
    """How much every row of the plain model's logits moves when what the sub-layers see of the stream is disturbed by about
    bfloat16's rounding (the larger of two draws): where a readout almost cancels and is normed to unit size, or a score
    stands near another, rounding alone moves a row by far more than elsewhere."""
    key = (model_dir, tuple(toks))
    if key not in _moves:
        import torch
        cfg, w = plain_model(model_dir)
        ref = plain_logits(model_dir, toks)
        out = np.zeros(len(toks))
        for seed in (1, 2):
            g = torch.Generator().manual_seed(seed)
            noise = lambda x: x * (1 + 2.0 ** -9 * torch.randn(x.shape, generator=g, dtype=x.dtype))
            moved = pg.logits(cfg, w, list(toks), noise).numpy()
            out = np.maximum(out, [row_error(moved[p], ref[p]) for p in range(len(toks))])
        _moves[key] = out
    return _moves[key]


def check_against_plain(model_dir, reqs, steps, outputs, dtype, vocab, label="", tol=None):
    """At most one row in two hundred (32-bit; bfloat16: one in fifty) may lie above the tolerance and none above five
    times it (with an explicit `tol`: none above it). A row's tolerance is at least four times what rounding (of bfloat16's
    size; in 32-bit 4,096 times smaller) moves the plain model's row by; in bfloat16 a token at
    which the plain model's router makes a close call is not compared, since rounding may rightly choose the other expert
    there, and neither are the CLOSE_REACH tokens behind it (32-bit compares every row)."""
    got = ru.collect(steps, outputs, vocab)
    strict = tol is not None
    tol = tol or TOL[dtype]
    worst, where, errs, skipped = 0.0, None, [], 0
    for rid, toks in reqs.items():
        ref = plain_logits(model_dir, toks)
        close = np.zeros(len(toks), dtype=bool)
        eased = np.ones(len(toks))
        if dtype == "bfloat16":
            at = closest_call(model_dir, toks) < CLOSE_CALL
            for pos in range(len(toks)):
                close[pos] = at[max(0, pos - CLOSE_REACH):pos + 1].any()
        if not strict:
            eased = np.maximum(1.0, 4 * moves(model_dir, toks) * (1.0 if dtype == "bfloat16" else 2.0 ** -12) / tol)
        assert sorted(got.get(rid, {})) == list(range(len(toks))), f"{rid}: positions missing"
        for pos in range(len(toks)):
            row = got[rid][pos]
            assert np.isfinite(row).all(), f"{label} {rid} position {pos}: non-finite logits"
            if close[pos]:
                skipped += 1
                continue
            e = row_error(row, ref[pos]) / eased[pos]
            errs.append(e)
            if e > worst:
                worst, where = e, (rid, pos)
    over = sum(e > tol for e in errs)
    print(f"worst difference from plain [{dtype} {label}]: {worst:.3e} at {where} (allowed {tol:.1e}; {over} of {len(errs)} rows above, {skipped} not compared)")
    if strict:
        assert worst <= tol, f"{label}: {where} differs by {worst:.3e} > {tol:.1e}"
    else:
        few = max(1, len(errs) // (50 if dtype == "bfloat16" else 200))
        assert worst <= 5 * tol and over <= few, f"{label}: {where} differs by {worst:.3e}, {over} of {len(errs)} rows above {tol:.1e}"
    return worst


def requests(vocab, lengths, seed):
    return ru.random_requests(vocab, lengths, seed=seed)


def decisive_requests(model_dir, vocab, lengths, seed):
    """Random requests without a close call of any router: a token at which the plain model makes one is drawn again (a
    wrong expert would be carried on by states and pages, so that nothing behind it could be compared in bfloat16)."""
    key = (model_dir, tuple(lengths), seed)
    if key not in _decisive:
        cfg, w = plain_model(model_dir)
        out = {}
        rng = np.random.default_rng(seed)
        for rid, toks in ru.random_requests(vocab, lengths, seed=seed).items():
            toks, at = list(toks), 0
            while at < len(toks):
                close = np.nonzero(pg.closest_call(cfg, w, toks[:at + 24]).numpy() < 2 * CLOSE_CALL)[0]
                if len(close) == 0:
                    at += 24
                    continue
                at = int(close[0])                 # (everything in front of it is settled: the model is causal)
                toks[at] = int(rng.integers(vocab))
            out[rid] = toks
        _decisive[key] = out
    return _decisive[key]
