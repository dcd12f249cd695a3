"""Small Zokunex configurations for the tests (none of them anyone's model), edits of their random weights that make a
fault visible, and the comparison of an engine's logits with the plain implementation's, position by position."""
from __future__ import annotations

import os
from typing import Dict

import numpy as np

import plain_zokunex as pz
import replay_util as ru


def mlstm(heads=3, dim=16, vdim=24, cap=9.0, mlp=None):
    m = {"heads": heads, "dim": dim, "gate_cap": cap}
    if vdim is not None:
        m["vdim"] = vdim
    return {"type": "mlstm", "mixer": m, "mlp": mlp}


def latent(heads=4, dim=16, rot_dim=8, vdim=24, kv_rank=32, base=5000.0, scale=None, mlp=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank,
         "scale": scale if scale is not None else (dim + rot_dim) ** -0.5}
    if rot_dim > 0:
        m["rot"] = {"base": base, "dims": rot_dim}
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def dense(ff=56):
    return {"kind": "dense", "ff": ff}


def moe(experts=4, identity=2, top=2, ff=24):
    r = {"experts": experts, "top": top}
    if identity is not None:
        r["identity"] = identity
    return {"kind": "moe", "router": r, "expert": {"ff": ff}}


def model(layers, vocab=300, width=64, eps=1e-5, logit_scale=0.5):
    c = {"architecture": "Zokunex", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if logit_scale is not None:
        c["logit_scale"] = logit_scale
    return c


# single mechanisms: each mixer alone without a feed-forward, each feed-forward behind a simple mixer
ONLY_MEMORY = model([mlstm()])
ONLY_MEMORY_SQUARE = model([mlstm(heads=1, dim=32, vdim=None, cap=4.0)], width=32, logit_scale=None)        # vdim as dim, one head
ONLY_MEMORY_ODD = model([mlstm(heads=2, dim=7, vdim=5, cap=20.0)], width=24)                                # no multiples of 4
ONLY_MEMORY_TILES = model([mlstm(heads=2, dim=72, vdim=136)], width=32)                                     # several key and value tiles
ONLY_MEMORY_SHARED = model([mlstm(heads=2, dim=160, vdim=256)], width=32)                                   # a head shared by workgroups in decoding
ONLY_MEMORY_WIDE = model([mlstm(heads=1, dim=72, vdim=576)], width=32)                                      # more value tiles than one workgroup takes
ONLY_MEMORY_WIDE_ODD = model([mlstm(heads=1, dim=9, vdim=331)], width=24)                                   # wide and unaligned
ONLY_MEMORY_UNALIGNED_KEYS = model([mlstm(heads=1, dim=10, vdim=300)], width=24)                            # aligned values beside unaligned keys
ONLY_MEMORY_BROAD = model([mlstm(heads=1, dim=8, vdim=8)], width=2056, vocab=64)                              # a stream wider than the norms keep in registers
ONLY_LATENT = model([latent()])
ONLY_LATENT_NO_TURN = model([latent(heads=3, dim=24, rot_dim=0, vdim=8, kv_rank=20)], width=48)
ONLY_LATENT_TURN_ONLY_LITTLE = model([latent(heads=2, dim=40, rot_dim=2, vdim=16, kv_rank=72, base=30.0)], width=32)
ONLY_LATENT_ONE_HEAD = model([latent(heads=1, dim=32, rot_dim=32, vdim=64, kv_rank=48)], width=40)
ONLY_LATENT_MANY = model([latent(heads=12, dim=8, rot_dim=4, vdim=12, kv_rank=16)], width=96)
ONLY_DENSE = model([mlstm(mlp=dense())])
ONLY_EXPERTS = model([mlstm(mlp=moe())])
EXPERTS_ALL = model([latent(mlp=moe(experts=3, identity=1, top=4, ff=16))], width=32)                       # every expert chosen
EXPERTS_NO_IDENTITY = model([latent(mlp=moe(experts=5, identity=None, top=3, ff=9))], width=32)
ONE_EXPERT = model([mlstm(mlp=moe(experts=1, identity=0, top=1, ff=32))], width=32)
MOSTLY_IDENTITY = model([mlstm(mlp=moe(experts=1, identity=5, top=3, ff=16))], width=32)
TOP_ONE = model([latent(mlp=moe(experts=6, identity=2, top=1, ff=16))], width=32)
# several layers in orders of their own
MIXED_A = model([
    latent(mlp=moe()),
    mlstm(mlp=dense(40)),
    mlstm(heads=2, dim=24, vdim=32, cap=15.0, mlp=moe(experts=6, identity=1, top=3, ff=16)),
    latent(heads=2, dim=32, rot_dim=16, vdim=32, kv_rank=48, base=900.0),
    mlstm(heads=1, dim=8, vdim=72, mlp=dense(72)),
], vocab=257, width=64, eps=1e-6, logit_scale=3.0)
MIXED_B = model([
    mlstm(heads=4, dim=8, vdim=12, cap=3.0),
    latent(heads=6, dim=8, rot_dim=8, vdim=16, kv_rank=24, mlp=dense(96)),
    latent(heads=3, dim=16, rot_dim=4, vdim=8, kv_rank=56, mlp=moe(experts=7, identity=3, top=4, ff=16)),
    mlstm(heads=2, dim=40, vdim=24, cap=25.0, mlp=moe(experts=3, identity=0, top=2, ff=24)),
], vocab=513, width=48, logit_scale=None)
# sizes that are multiples of neither 8 nor 4; a width that is odd
ODD = model([
    mlstm(heads=3, dim=10, vdim=7, mlp=moe(experts=5, identity=2, top=2, ff=13)),
    latent(heads=3, dim=6, rot_dim=2, vdim=9, kv_rank=11, mlp=dense(19)),
    mlstm(heads=1, dim=5, vdim=9, mlp=moe(experts=3, identity=1, top=3, ff=9)),
    latent(heads=2, dim=7, rot_dim=6, vdim=5, kv_rank=17),
], vocab=101, width=43)
# the sizes of a larger model's layers
LARGER = model([
    mlstm(heads=4, dim=64, vdim=64, mlp=moe(experts=6, identity=2, top=2, ff=96)),
    latent(heads=4, dim=64, rot_dim=32, vdim=64, kv_rank=128, mlp=dense(384)),
    mlstm(heads=2, dim=128, vdim=192, mlp=dense(320)),
    latent(heads=8, dim=32, rot_dim=64, vdim=48, kv_rank=224, mlp=moe(experts=6, identity=2, top=4, ff=96)),
], vocab=211, width=256)
# scores that single keys dominate
PEAKED = model([latent(scale=1.5), latent(heads=2, dim=8, rot_dim=16, vdim=16, kv_rank=24, scale=1.2, base=200.0)], width=32)
PEAKED_TILES = model([latent(heads=4, dim=32, rot_dim=32, vdim=32, kv_rank=64, scale=0.9)], width=64)
# a memory that keeps everything, written by tokens whose input gates differ by orders of magnitude: what a token far back
# wrote carries late rows (with KEEPING's edits)
KEEPING = model([mlstm(heads=2, dim=16, vdim=16, cap=8.0)], width=32)
# memories that hard resets empty every few tokens, beside long stretches that keep everything (with RESETTING's edits)
RESETTING = model([mlstm(heads=3, dim=16, vdim=20, cap=15.0)], width=32)
# input gates so small that the normaliser's lower bound decides (with FAINT's edits)
FAINT = model([mlstm(heads=2, dim=16, vdim=16, cap=12.0)], width=32)

# without routed experts (greedy generation in bfloat16: what is generated cannot be chosen to suit a router)
UNROUTED = model([mlstm(mlp=dense(48)), latent(), mlstm(heads=2, dim=24, vdim=16, cap=15.0, mlp=dense(40)),
                  latent(heads=2, dim=32, rot_dim=16, vdim=32, kv_rank=48, mlp=dense(40))], vocab=257, logit_scale=2.0)

# name -> tensor name -> (factor, added): the stored tensor times factor plus added
EDITS = {
    "KEEPING": {"l0.mix.i": (4.0, 0.0), "l0.mix.f": (0.25, 0.0), "l0.mix.f.b": (0.0, 7.5)},
    "RESETTING": {"l0.mix.f": (14.0, 0.0), "l0.mix.f.b": (0.0, 6.0), "l0.mix.i": (4.0, 0.0)},
    # (scores further apart: fewer tokens at which rounding may choose another expert)
    "MIXED_A": {"l0.mlp.router": (3.0, 0.0), "l2.mlp.router": (3.0, 0.0)},
    "MIXED_B": {"l2.mlp.router": (3.0, 0.0), "l3.mlp.router": (3.0, 0.0)},
    "ODD": {"l0.mlp.router": (3.0, 0.0), "l2.mlp.router": (3.0, 0.0)},
    "FAINT": {"l0.mix.i.b": (0.0, -7.0), "l0.mix.f.b": (0.0, 4.0), "l0.mix.i": (2.0, 0.0)},
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
TOL = {"float32": 2e-5, "bfloat16": 6e-2}
TOL_PEAKED = 1e-4

_plain: Dict[tuple, np.ndarray] = {}
_weights: Dict[str, tuple] = {}
def strong_tokens(model_dir, n):
    """The n token ids that write most strongly into the first layer's memory (a first layer's gates depend on the token
    alone), the strongest first."""
    cfg, w = plain_model(model_dir)
    i, _ = pz.mlstm_gates(w["embed"], w, "l0.mix.", cfg["layers"][0]["mixer"]["gate_cap"])
    return [int(t) for t in i.min(dim=1).values.argsort(descending=True)[:n]]


_calls: Dict[tuple, np.ndarray] = {}
CLOSE_CALL = 0.006      # a gap between two choice scores below which bfloat16 rounding may choose the other expert
CLOSE_REACH = 8         # positions behind such a token that still carry it most


def plain_model(model_dir):
    if model_dir not in _weights:
        _weights[model_dir] = pz.read_model(model_dir)
    return _weights[model_dir]


def plain_logits(model_dir, toks) -> np.ndarray:
    key = (model_dir, tuple(toks))
    if key not in _plain:
        cfg, w = plain_model(model_dir)
        _plain[key] = pz.logits(cfg, w, list(toks)).numpy()
    return _plain[key]


def closest_call(model_dir, toks) -> np.ndarray:
    key = (model_dir, tuple(toks))
    if key not in _calls:
        cfg, w = plain_model(model_dir)
        _calls[key] = pz.closest_call(cfg, w, list(toks)).numpy()
    return _calls[key]


def row_error(got, ref) -> float:
    d = got.astype(np.float64) - ref
    d = d - d.mean()
    r = ref - ref.mean()
    return float(np.sqrt((d * d).mean()) / np.sqrt((r * r).mean()))


_moves: Dict[tuple, np.ndarray] = {}


def moves(model_dir, toks) -> np.ndarray:
    """How much every row of the plain model's logits moves when what the sub-layers see of the stream is disturbed by about
    bfloat16's rounding (the larger of two draws): where a memory's readout almost cancels and is normed to unit size, or a
    key's product with a query is near zero, rounding alone moves a row by far more than elsewhere."""
    key = (model_dir, tuple(toks))
    if key not in _moves:
        import torch
        cfg, w = plain_model(model_dir)
        ref = plain_logits(model_dir, toks)
        out = np.zeros(len(toks))
        for seed in (1, 2):
            g = torch.Generator().manual_seed(seed)
            noise = lambda x: x * (1 + 2.0 ** -9 * torch.randn(x.shape, generator=g, dtype=x.dtype))
            moved = pz.logits(cfg, w, list(toks), noise).numpy()
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
    worst, where, errs = 0.0, None, []
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
                continue
            e = row_error(row, ref[pos]) / eased[pos]
            errs.append(e)
            if e > worst:
                worst, where = e, (rid, pos)
    over = sum(e > tol for e in errs)
    print(f"worst difference from plain [{dtype} {label}]: {worst:.3e} at {where} (allowed {tol:.1e}; {over} of {len(errs)} rows above)")
    if strict:
        assert worst <= tol, f"{label}: {where} differs by {worst:.3e} > {tol:.1e}"
    else:
        few = max(1, len(errs) // (50 if dtype == "bfloat16" else 200))
        assert worst <= 5 * tol and over <= few, f"{label}: {where} differs by {worst:.3e}, {over} of {len(errs)} rows above {tol:.1e}"
    return worst


def requests(vocab, lengths, seed):
    return ru.random_requests(vocab, lengths, seed=seed)


_decisive: Dict[tuple, dict] = {}


def decisive_requests(model_dir, vocab, lengths, seed):
    """Random requests without a close call of any router: a token at which the plain model makes one is drawn again (a
    wrong expert would be carried on by the memories, so that nothing behind it could be compared in bfloat16)."""
    key = (model_dir, tuple(lengths), seed)
    if key not in _decisive:
        cfg, w = plain_model(model_dir)
        out = {}
        rng = np.random.default_rng(seed)
        for rid, toks in ru.random_requests(vocab, lengths, seed=seed).items():
            toks, at = list(toks), 0
            while at < len(toks):
                close = np.nonzero(pz.closest_call(cfg, w, toks[:at + 24]).numpy() < 2 * CLOSE_CALL)[0]
                if len(close) == 0:
                    at += 24
                    continue
                at = int(close[0])                 # (everything in front of it is settled: the model is causal)
                toks[at] = int(rng.integers(vocab))
            out[rid] = toks
        _decisive[key] = out
    return _decisive[key]
