"""Gisedra without a GPU: what its configuration asks of a checkpoint, what it refuses, the plain implementation's own
consistency (closed forms of the single mechanisms), and that the cases of the GPU tests would show a window, kept position,
rotation, convolution, decay, router, loop or token input that is off."""
import copy
import math

import pytest
import torch

import gisedra_cases as gc
import plain_gisedra as pg
from mini_llm_amd import check_model_dir, describe_config, registered_architectures, write_random_model
from mini_llm_amd.config import ConfigError

F64 = torch.float64


def test_registered_and_tensors_follow_the_layer_list():
    assert "Gisedra" in registered_architectures()
    d = describe_config(gc.MIXED_A)
    assert d["architecture"] == "Gisedra"
    shapes = {t["name"]: t["shape"] for t in d["tensors"]}
    assert shapes["embed"] == [257, 64] and shapes["head"] == [257, 64] and shapes["loop.step"] == [2, 64]
    # the second table holds every layer's columns, looped layers once
    assert shapes["side.embed"] == [257, 64] and shapes["l3.side.gate"] == [16, 64] and shapes["l3.side.proj"] == [64, 16] and shapes["l3.side.norm"] == [64]
    # a norm has a weight, a bias and one number
    assert shapes["l0.norm1"] == [64] and shapes["l0.norm1b.b"] == [64] and shapes["final.norm.alpha"] == []
    # the pair: grouped heads with values of their own width, taps per channel, one gate row per value column; retention
    assert shapes["l0.mix.left.q"] == [64, 64] and shapes["l0.mix.left.k"] == [32, 64] and shapes["l0.mix.left.v"] == [48, 64]
    assert shapes["l0.mix.left.q.conv"] == [64, 3] and shapes["l0.mix.left.v.conv"] == [48, 3] and shapes["l2.mix.left.k.conv"] == [32, 4]
    assert shapes["l0.mix.left.g"] == [96, 64] and shapes["l0.mix.left.o"] == [64, 96]
    assert shapes["l2.mix.right.q"] == [48, 64] and shapes["l2.mix.right.v"] == [24, 64] and shapes["l2.mix.right.g"] == [24, 64] and shapes["l2.mix.right.o"] == [64, 24]
    # latent attention without a query latent
    assert shapes["l3.mix.q"] == [96, 64] and shapes["l3.mix.dkv"] == [64, 64] and shapes["l3.mix.dkv.norm"] == [48]
    assert shapes["l3.mix.uk"] == [64, 48] and shapes["l3.mix.uv"] == [64, 48] and shapes["l3.mix.o"] == [64, 64]
    assert shapes["l1.mlp.router"] == [7, 64] and shapes["l1.mlp.router.b"] == [7] and shapes["l1.mlp.e6.gate"] == [16, 64] and shapes["l1.mlp.e6.down"] == [64, 16]
    # no feed-forward: no second pair of norms
    assert "l2.norm2" not in shapes and "l2.norm2b.alpha" not in shapes and "l2.mlp.router" not in shapes and shapes["l2.norm1b"] == [64]
    roles = {t["name"]: t["role"] for t in d["tensors"]}
    assert roles["l0.mix.left.q.conv"] == "vector" and roles["l1.mlp.router.b"] == "vector" and roles["side.embed"] == "matrix" and roles["loop.step"] == "vector"


def test_keys_that_may_be_absent_have_the_plain_meaning():
    cfg = copy.deepcopy(gc.MIXED_A)
    cfg.pop("loop")
    cfg["token_side"] = None
    left = cfg["layers"][0]["mixer"]["left"]
    for key in ("kv_heads", "vdim", "conv", "rot", "mask"):
        left.pop(key)
    cfg["layers"][0]["mixer"].pop("left_scale")
    cfg["layers"][0]["mixer"]["right"].pop("vdim")
    for key in ("rot_dim", "rot", "mask"):
        cfg["layers"][1]["mixer"].pop(key)
    cfg["layers"][1]["mlp"].pop("kind")
    cfg["layers"][3].pop("mlp")
    shapes = {t["name"]: t["shape"] for t in describe_config(cfg)["tensors"]}
    assert shapes["l0.mix.left.k"] == [64, 64] and shapes["l0.mix.left.v"] == [64, 64] and "l0.mix.left.q.conv" not in shapes
    assert shapes["l0.mix.right.v"] == [16, 64] and shapes["l1.mix.q"] == [64, 64] and shapes["l1.mix.dkv"] == [32, 64]
    assert not any(n.startswith(("side.", "loop.")) or ".side." in n for n in shapes) and "l3.norm2" not in shapes and "l1.mlp.router" in shapes


@pytest.mark.parametrize("change, message", [
    (lambda c: c["layers"][1].__setitem__("type", "lstm"), "unknown layer type"),
    (lambda c: c["layers"][0]["mixer"].pop("right"), "right"),
    (lambda c: c["layers"][0]["mixer"]["right"].__setitem__("decay", [0.5]), "decay"),
    (lambda c: c["layers"][0]["mixer"]["right"].__setitem__("decay", [0.5, 0.0]), "decay"),
    (lambda c: c["layers"][0]["mixer"]["right"].__setitem__("decay", [0.5, 1.5]), "decay"),
    (lambda c: c["layers"][0]["mixer"]["left"].__setitem__("kv_heads", 3), "multiple"),
    (lambda c: c["layers"][0]["mixer"]["left"].__setitem__("conv", 17), "16 taps"),
    (lambda c: c["layers"][0]["mixer"]["left"]["rot"].__setitem__("dims", 5), "even"),
    (lambda c: c["layers"][0]["mixer"]["left"]["rot"].__setitem__("dims", 18), "at most"),
    (lambda c: c["layers"][0]["mixer"]["left"]["rot"]["scaling"].__setitem__("high", 0.5), "high above low"),
    (lambda c: c["layers"][0]["mixer"]["left"]["rot"]["scaling"].pop("factor"), "factor"),
    (lambda c: c["layers"][0]["mixer"]["left"]["mask"].__setitem__("size", 0), "size"),
    (lambda c: c["layers"][0]["mixer"]["left"]["mask"].__setitem__("keep_first", -1), "keep_first"),
    (lambda c: c["layers"][1]["mixer"]["mask"].__setitem__("keep_first", 2), "keeps no first"),
    (lambda c: c["layers"][1]["mixer"]["rot"].__setitem__("scaling", gc.SCALING), "not scaled"),
    (lambda c: c["layers"][1]["mixer"].pop("scale"), "scale"),
    (lambda c: c["layers"][1]["mixer"].pop("kv_rank"), "kv_rank"),
    (lambda c: c["layers"][1]["mlp"]["router"].__setitem__("top", 8), "top"),
    (lambda c: c["layers"][1]["mlp"]["router"].__setitem__("experts", 300), "256"),
    (lambda c: c["layers"][1]["mlp"].__setitem__("kind", "dense"), "moe"),
    (lambda c: c["loop"].__setitem__("stop", 9), "loop"),
    (lambda c: c["loop"].__setitem__("times", 0), "times"),
    (lambda c: c["token_side"].pop("dim"), "dim"),
    (lambda c: c.pop("norm"), "norm"),
])
def test_refusals(change, message):
    cfg = copy.deepcopy(gc.MIXED_A)
    change(cfg)
    with pytest.raises(ConfigError, match=message):
        describe_config(cfg)


def test_written_folder_checks(tmp_path):
    d = write_random_model(dict(gc.MIXED_B), str(tmp_path / "m"), 1)
    arch, n_tensors, _ = check_model_dir(d)
    assert arch == "Gisedra" and n_tensors == len(describe_config(gc.MIXED_B)["tensors"])
    cfg, w = pg.read_model(d)
    assert pg.logits(cfg, w, [1, 2, 3, 4, 5]).shape == (5, 513)
    assert pg.streams(cfg, w, [1, 2]).shape == (5, 2, 48)          # (two layers twice, then the third)
    assert check_model_dir(gc.write_case("MIXED_A", str(tmp_path / "edited")))[0] == "Gisedra"


# -- the plain mechanisms against closed forms -----------------------------------------------------------
def test_dynamic_tanh_has_no_statistics():
    w = {"n": torch.tensor([2.0, 1.0], dtype=F64), "n.b": torch.tensor([0.5, 0.0], dtype=F64), "n.alpha": torch.tensor(0.5, dtype=F64)}
    y = pg.dynamic_tanh(torch.tensor([[1.0, 100.0], [0.0, -2.0]], dtype=F64), w, "n")
    assert math.isclose(float(y[0, 0]), 2 * math.tanh(0.5) + 0.5) and float(y[0, 1]) == 1.0
    assert float(y[1, 0]) == 0.5 and math.isclose(float(y[1, 1]), math.tanh(-1.0))


def test_the_last_tap_is_the_tokens_own():
    u = torch.arange(1.0, 6.0, dtype=F64)[:, None]
    y = pg.short_conv(u, torch.tensor([[100.0, 10.0, 1.0]], dtype=F64))
    assert y[:, 0].tolist() == [1.0, 12.0, 123.0, 234.0, 345.0]
    assert torch.equal(pg.short_conv(u[:1], torch.tensor([[100.0, 10.0, 1.0]], dtype=F64)), u[:1])


def test_frequencies_are_kept_stretched_or_blended():
    rot = {"base": 10000.0, "dims": 64, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 256}}
    f, plain = pg.frequencies(rot), pg.frequencies({"base": 10000.0, "dims": 64})
    kinds = set()
    for a, b in zip(f, plain):
        turn = 2 * math.pi / b
        if turn < 64:
            assert a == b
            kinds.add("kept")
        elif turn > 256:
            assert a == b / 8
            kinds.add("stretched")
        else:
            assert b / 8 < a < b
            kinds.add("between")
    assert kinds == {"kept", "stretched", "between"}
    # at the two borders the blend meets both
    edge = lambda turn: (256 / turn - 1.0) / 3.0
    assert edge(64) == 1.0 and edge(256) == 0.0


def test_turns_pair_halves_or_neighbours_and_keep_lengths():
    v = torch.randn(7, 2, 8, dtype=F64)
    for interleaved in (False, True):
        out = pg.turn(v, {"base": 100.0, "dims": 6}, interleaved)
        assert torch.allclose(out.norm(dim=-1), v.norm(dim=-1)) and torch.equal(out[..., 6:], v[..., 6:]) and torch.equal(out[0], v[0])
    one = torch.zeros(4, 8, dtype=F64)
    one[3, 2] = 1.0
    a, b = 3 * 100.0 ** (-4.0 / 6), 3 * 100.0 ** (-2.0 / 6)
    half, near = pg.turn(one, {"base": 100.0, "dims": 6}, False)[3], pg.turn(one, {"base": 100.0, "dims": 6}, True)[3]
    assert math.isclose(float(half[2]), math.cos(a)) and math.isclose(float(half[5]), math.sin(a))
    assert math.isclose(float(near[2]), math.cos(b)) and math.isclose(float(near[3]), math.sin(b))


def test_who_sees_whom():
    see = pg.visible(8, {"size": 3, "keep_first": 2})
    assert see[7].tolist() == [True, True, False, False, False, True, True, True]
    assert see[3].tolist() == [True, True, True, True] + [False] * 4 and see[0].tolist() == [True] + [False] * 7
    assert pg.visible(5, {"size": 1}).equal(torch.eye(5, dtype=torch.bool)) and pg.visible(4, None).equal(torch.ones(4, 4, dtype=torch.bool).tril())


def test_retention_is_a_decayed_sum():
    g = torch.Generator().manual_seed(2)
    q, k, v = (torch.randn(6, n, generator=g, dtype=F64) for n in (3, 3, 4))
    out = pg.retention_readout(q, k, v, 0.75)
    for t in range(6):
        ref = sum(0.75 ** (t - s) * float(q[t] @ k[s]) * v[s] for s in range(t + 1))
        assert torch.allclose(out[t], ref)


def test_experts_are_weighed_over_the_chosen_only():
    z = torch.tensor([[0.0, math.log(3.0), -9.0, 0.0]], dtype=F64)
    assert pg.chosen_experts(z, 2) == [[1, 0]]                      # (the lower index wins a tie)
    w = {"router": torch.zeros(4, 1, dtype=F64), "router.b": z[0]}
    for e in range(4):
        w.update({f"e{e}.gate": torch.ones(1, 1, dtype=F64), f"e{e}.up": torch.ones(1, 1, dtype=F64), f"e{e}.down": torch.full((1, 1), float(10 ** e), dtype=F64)})
    y = pg.routed_experts(torch.ones(1, 1, dtype=F64), w, "", {"router": {"experts": 4, "top": 2}})
    one = 1 / (1 + math.exp(-1.0))                                  # silu(1) * 1
    assert math.isclose(float(y), one * (0.75 * 10 + 0.25 * 1))


def test_passes_and_their_sums():
    cfg = gc.model([gc.latent(), gc.latent(), gc.latent()], loop=(1, 2, 3))
    assert pg.order(cfg) == [(0, None), (1, 0), (1, 1), (1, 2), (2, None)]
    w = {"loop.step": torch.tensor([[1.0], [2.0]], dtype=F64)}
    x, x0 = torch.tensor([[10.0]], dtype=F64), torch.tensor([[100.0]], dtype=F64)
    assert float(pg.before_pass(x, x0, w, 0)) == 11.0 and float(pg.before_pass(x, x0, w, 1)) == 112.0


@pytest.mark.parametrize("what, name", [
    ("window", "PEAKED"), ("latent_window", "PEAKED"), ("keep_first", "PEAKED"), ("kept_distance", "PEAKED"), ("lost_key", "PEAKED"), ("scaling", "PEAKED"),
    ("angle", "PEAKED"), ("pairs", "PEAKED"), ("taps_shift", "PEAKED"), ("values_unconvolved", "PEAKED"), ("lost_conv", "PEAKED"), ("gate", "ONLY_PAIR"),
    ("scales", "ONLY_PAIR"), ("first_token", "SLOW"), ("lost_state", "SLOW"), ("decay", "SLOW"), ("head_norm", "SLOW"), ("router_bias", "ONLY_EXPERTS"),
    ("over_all", "ONLY_EXPERTS"), ("side_columns", "ONLY_SIDE"), ("side_token", "ONLY_SIDE"), ("no_embedding", "LOOP_ALL"), ("step", "LOOP_ALL"), ("pass_state", "LOOP_ALL"),
    ("alpha", "MIXED_A")])
def test_the_cases_have_teeth(tmp_path, what, name, monkeypatch):
    """The plain model with one mistake differs from the plain model by far more than the tolerance in many late rows: the
    GPU tests would show such a fault."""
    d = gc.write_case(name, str(tmp_path / "m"))
    cfg, w = pg.read_model(d)
    n = 120
    toks = gc.requests(cfg["vocab"], [n], seed=21)["r0"]
    a = pg.logits(cfg, w, toks).numpy()
    off, toks_b, w_b = copy.deepcopy(cfg), list(toks), dict(w)
    pairs = [l["mixer"] for l in off["layers"] if l["type"] == "parallel"]
    latents = [l["mixer"] for l in off["layers"] if l["type"] == "latent_attention"]
    if what == "window":
        pairs[0]["left"]["mask"]["size"] += 1
    elif what == "latent_window":
        latents[0]["mask"]["size"] -= 1
    elif what == "keep_first":
        pairs[0]["left"]["mask"]["keep_first"] -= 1
    elif what == "kept_distance":                    # kept keys turned as if they stood right in front of the window
        def moved(v, rot, interleaved):
            out = turn(v, rot, interleaved)
            if not interleaved and v.shape[1] == 2:                  # (the keys' heads)
                late = torch.cat([v[:3], v[3:]])
                out[:3] = turn(torch.cat([late[:3]] * 34), rot, interleaved)[99:102]
            return out
        turn = pg.turn
        monkeypatch.setattr(pg, "turn", moved)
    elif what == "lost_key":
        def visible(T, mask):
            see = seen(T, mask).clone()
            see[100:, 95] = False
            return see
        seen = pg.visible
        monkeypatch.setattr(pg, "visible", visible)
    elif what == "scaling":
        pairs[0]["left"]["rot"].pop("scaling")
    elif what == "angle":
        latents[0]["rot"]["base"] *= 1.1
    elif what == "pairs":
        turn = pg.turn
        monkeypatch.setattr(pg, "turn", lambda v, rot, interleaved: turn(v, rot, not interleaved))
    elif what == "taps_shift":
        for t in ("q", "k", "v"):
            w_b[f"l0.mix.left.{t}.conv"] = w[f"l0.mix.left.{t}.conv"].flip(1)
    elif what == "values_unconvolved":
        w_b["l0.mix.left.v.conv"] = torch.tensor([0.0, 0.0, 1.0], dtype=F64).expand_as(w["l0.mix.left.v.conv"])
    elif what == "lost_conv":                        # as if a portion that begins at 64 found no carried rows
        conv = pg.short_conv
        monkeypatch.setattr(pg, "short_conv", lambda u, taps: torch.cat([conv(u[:64], taps), conv(u[64:], taps)]))
    elif what == "gate":
        w_b["l0.mix.left.g"] = w["l0.mix.left.g"] * 0.7
    elif what == "scales":
        pairs[0]["left_scale"], pairs[0]["right_scale"] = pairs[0]["right_scale"], pairs[0]["left_scale"]
    elif what == "first_token":
        toks_b[0] = (toks_b[0] + 1) % cfg["vocab"]
    elif what == "lost_state":
        readout = pg.retention_readout
        monkeypatch.setattr(pg, "retention_readout", lambda q, k, v, f: torch.cat([readout(q[:64], k[:64], v[:64], f), readout(q[64:], k[64:], v[64:], f)]))
    elif what == "decay":
        pairs[0]["right"]["decay"][0] = 1.0
    elif what == "head_norm":
        rms = pg.unit_rms
        monkeypatch.setattr(pg, "unit_rms", lambda x, eps: rms(x.reshape(x.shape[0], -1), eps).reshape(x.shape))
    elif what == "router_bias":
        w_b["l0.mlp.router.b"] = w["l0.mlp.router.b"] * 0
    elif what == "over_all":
        softmax = torch.softmax
        z_all = {}

        def logits_kept(h, ww, pre):
            z_all["z"] = h @ ww[pre + "router"].T + ww[pre + "router.b"]
            z_all["t"] = 0
            return z_all["z"]

        def over_all(z, dim):
            if z.dim() != 1:
                return softmax(z, dim=dim)
            t = z_all["t"]
            z_all["t"] += 1
            return torch.exp(z - torch.logsumexp(z_all["z"][t], dim=0))
        monkeypatch.setattr(pg, "router_logits", logits_kept)
        monkeypatch.setattr(torch, "softmax", over_all)
    elif what == "side_columns":                     # every layer reads the first one's columns
        side = pg.token_side

        def first_columns(x, ww, i, tokens, dim, eps):
            return side(x, {**ww, "side.embed": torch.cat([ww["side.embed"][:, :dim]] * 2, dim=1)}, i, tokens, dim, eps)
        monkeypatch.setattr(pg, "token_side", first_columns)
    elif what == "side_token":                       # the token in front in place of the token itself
        side = pg.token_side
        monkeypatch.setattr(pg, "token_side", lambda x, ww, i, tokens, dim, eps: side(x, ww, i, [tokens[0]] + tokens[:-1], dim, eps))
    elif what == "no_embedding":
        monkeypatch.setattr(pg, "before_pass", lambda x, x0, ww, t: x + ww["loop.step"][t])
    elif what == "step":
        w_b["loop.step"] = w["loop.step"].flip(0)
    elif what == "pass_state":                       # as if the passes shared one memory: the second finds the first one's
        readout, kept = pg.retention_readout, {}

        def shared(q, k, v, f):
            key = (float(f), q.shape[1])
            before = kept.get(key)
            kept[key] = (k, v)
            if before is None:
                return readout(q, k, v, f)
            return readout(torch.cat([before[0], q]), torch.cat([before[0], k]), torch.cat([before[1], v]), f)[q.shape[0]:]
        monkeypatch.setattr(pg, "retention_readout", shared)
    elif what == "alpha":
        w_b["l1.norm2b.alpha"] = w["l1.norm2b.alpha"] * 1.05
    b = pg.logits(off, w_b, toks_b).numpy()
    late = range(n - 50, n) if what != "lost_key" else range(100, 115)
    if what == "lost_conv":
        late = range(64, 66)
    errs = [gc.row_error(b[p], a[p]) for p in late]
    floor = 10 * (gc.TOL_PEAKED if name == "PEAKED" else gc.TOL["float32"])
    share = 0.12 if what in ("lost_key", "keep_first", "window", "latent_window", "kept_distance") else 0.5
    assert sum(e > floor for e in errs) > share * len(errs), sorted(errs)
