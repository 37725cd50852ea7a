"""The Gosavik architecture on the host: its configuration and spec, the plain implementation's mechanisms against closed
forms, and the engine (step function, cache manager, scheduler, generate) on the torch stand-ins for the kernels against
the plain implementation, in 32-bit."""
import copy
import math

import pytest
import torch

import gosavik_models as GM
import helpers as H
import plain_gosavik as pg
from torch_ops import TorchOps
from tiny_inference_server_amd.config import ARCHITECTURES, ConfigError, config_from_dict, load_config
from tiny_inference_server_amd.engine import Engine
from tiny_inference_server_amd.engine.generate import generate
from tiny_inference_server_amd.parts.attention import slowed_frequencies
from tiny_inference_server_amd.parts.spec import PagedKvNeed, StateNeed
from tiny_inference_server_amd.weights.loader import spec_tensors

TOL32 = 3e-5
F64 = torch.float64


def model(name, seed=5):
    cfg = GM.CONFIGS[name]
    w = GM.random_weights(cfg, seed)
    return cfg, w, GM.as_f64(w)


def engine_for(cfg, w, **kw):
    kw.setdefault("max_requests", 4)
    kw.setdefault("page_size", 8)
    kw.setdefault("max_tokens", 640)
    return Engine(config=config_from_dict(cfg), tensors={n: t.float() for n, t in w.items()}, dtype="float32",
                  ops=TorchOps(graphs=kw.pop("graphs", False)), **kw)


# ---- configuration and spec ------------------------------------------------------------------------------------

def test_spec_names_every_tensor_and_every_pass_has_its_own_cache(tmp_path):
    for name, cfg in GM.CONFIGS.items():
        w = GM.random_weights(cfg, 1)
        folder = GM.write_folder(str(tmp_path / name), cfg, w)
        c = load_config(folder)
        assert c.architecture == "Gosavik" and c.to_dict() == config_from_dict(c.to_dict()).to_dict()
        spec = ARCHITECTURES.get(c.architecture).build_spec(c)
        assert spec_tensors(spec) == {n: tuple(t.shape) for n, t in w.items()}
        order = pg.run_order(len(cfg["layers"]), cfg.get("loop"))
        assert [call.layer for call in spec.stages[0].calls] == order
        needs = engine_for(cfg, w).model.cache_needs()
        for i, layer in enumerate(order):
            m, latent = cfg["layers"][layer]["mixer"], cfg["layers"][layer]["type"] == "latent_attention"
            assert needs[f"trunk.{i}:mixer_shift"] == StateNeed((cfg["width"],), "float32")
            pages = needs[f"trunk.{i}:mixer"]
            assert isinstance(pages, PagedKvNeed) and pages.window == (m.get("mask") or {}).get("size", 0)
            kept = needs.get(f"trunk.{i}:mixer.state")
            if latent or m["conv"] == 1:
                assert kept is None
            else:
                assert kept.shape == ((m["conv"] - 1) * (m["heads"] * m["dim"] + m["kv_heads"] * (m["dim"] + m["vdim"])),)


def test_a_layer_without_a_feed_forward_may_carry_what_stands_around_one(tmp_path):
    cfg, w, _ = model("A")
    extra = {**w, "l3.norm2": w["l3.norm1"].clone(), **{f"l3.hc2.{k}": w[f"l3.hc1.{k}"].clone() for k in ("in", "out", "mix")}}
    folder = GM.write_folder(str(tmp_path / "m"), cfg, extra)
    assert Engine(folder, dtype="float32", max_tokens=64, ops=TorchOps()).step([("a", [1, 2], [1])]).logits.shape == (1, cfg["vocab"])


def test_configuration_errors_name_the_key():
    good = GM.CONFIGS["A"]
    for path, value, word in [(("layers", 0, "type"), "parallel", "type"), (("layers", 1, "mixer", "kv_heads"), 3, "kv_heads"),
                              (("layers", 0, "mixer", "rot", "dims"), 3, "rot.dims"), (("layers", 0, "mixer", "rot", "dims"), 10, "rot.dims"),
                              (("layers", 0, "mixer", "rot", "scaling", "fast"), 0.0, "scaling"),
                              (("layers", 0, "mixer", "mask", "size"), 0, "size"), (("layers", 0, "mixer", "q_rank"), 0, "q_rank"),
                              (("layers", 1, "mixer", "vdim"), 7, "vdim"), (("layers", 1, "mixer", "conv"), 0, "conv"),
                              (("layers", 1, "mixer", "rot"), None, "rot.base"), (("layers", 0, "mlp", "kind"), "gated", "mlp"),
                              (("loop", "stop"), 5, "loop"), (("loop", "times"), 0, "times"), (("streams",), 0, "streams"),
                              (("norm",), {}, "eps")]:
        bad = copy.deepcopy(good)
        d = bad
        for k in path[:-1]:
            d = d[k]
        d[path[-1]] = value
        with pytest.raises(ConfigError, match=word):
            config_from_dict(bad)


# ---- the plain implementation's mechanisms against closed forms ----------------------------------------------------

def test_plain_streams_and_shift():
    g = torch.Generator().manual_seed(0)
    X, y = torch.randn(3, 4, 5, generator=g, dtype=F64), torch.randn(4, 5, generator=g, dtype=F64)
    read, out, mix = (torch.randn(s, generator=g, dtype=F64) for s in ((3,), (3,), (3, 3)))
    u, Z = pg.read_streams(X, read), pg.write_streams(X, mix, out, y)
    for t in range(4):
        assert torch.allclose(u[t], sum(read[s] * X[s, t] for s in range(3)))
        for to in range(3):
            assert torch.allclose(Z[to, t], sum(mix[s, to] * X[s, t] for s in range(3)) + out[to] * y[t])
    h, a = torch.randn(4, 5, generator=g, dtype=F64), torch.rand(5, generator=g, dtype=F64)
    m = pg.token_shift(h, a)
    assert torch.allclose(m[0], h[0] * (1 - a)) and torch.allclose(m[3], h[3] * (1 - a) + h[2] * a)
    assert torch.equal(pg.token_shift(h, torch.zeros(5, dtype=F64)), h)
    assert pg.run_order(5, {"start": 1, "stop": 3, "times": 3}) == [0, 1, 2, 1, 2, 1, 2, 3, 4]
    assert pg.run_order(3, None) == [0, 1, 2]


def test_plain_rotations_and_slowed_waves():
    g = torch.Generator().manual_seed(1)
    sc = {"factor": 4.0, "original": 64, "fast": 8.0, "slow": 1.0}
    f0 = pg.frequencies(16, 100.0)
    f, factor = pg.slowed(16, 100.0, sc)
    # pairs that turn more than `fast` times in `original` positions are kept, fewer than `slow` times divided
    turns = 64 * f0 / (2 * math.pi)
    assert torch.equal(f[turns > 8.0], f0[turns > 8.0]) and (turns > 8.0).any()
    assert torch.allclose(f[turns < 0.7], f0[turns < 0.7] / 4.0) and (turns < 0.7).any()
    assert ((f < f0 * 0.999) & (f > f0 / 3.999)).any() and abs(factor - (0.1 * math.log(4.0) + 1)) < 1e-14
    e, ef = slowed_frequencies(16, 100.0, 4.0, 64, 8.0, 1.0)       # the engine's table, written another way
    assert torch.allclose(e, f, rtol=1e-13) and abs(ef - factor) < 1e-14
    # where the two ends fall together the ramp is a step
    e, _ = slowed_frequencies(8, 1e6, 3.0, 40, 2.0, 2.0)
    assert torch.allclose(e, pg.slowed(8, 1e6, {"factor": 3.0, "original": 40, "fast": 2.0, "slow": 2.0})[0], rtol=1e-13)
    x, y = torch.randn(1, 1, 10, generator=g, dtype=F64), torch.randn(1, 1, 10, generator=g, dtype=F64)
    fr = pg.frequencies(6, 50.0)
    for turn in (pg.rotate_half, pg.rotate_pairs):
        s = [float((turn(x, torch.tensor([p + 2]), 6, fr) * turn(y, torch.tensor([p]), 6, fr)).sum()) for p in (1, 8, 38)]
        assert abs(s[0] - s[1]) < 1e-12 and abs(s[0] - s[2]) < 1e-12           # the distance alone counts
        z = turn(turn(x, torch.tensor([7]), 6, fr), torch.tensor([-7]), 6, fr)
        assert torch.allclose(z, x, atol=1e-13) and torch.equal(turn(x, torch.tensor([7]), 6, fr)[..., 6:], x[..., 6:])
    a = 7 * 50.0 ** (-2.0 / 6)
    h, p = pg.rotate_half(x, torch.tensor([7]), 6, fr, 1.5)[0, 0], pg.rotate_pairs(x, torch.tensor([7]), 6, fr, 1.5)[0, 0]
    assert torch.isclose(h[1], 1.5 * (x[0, 0, 1] * math.cos(a) - x[0, 0, 4] * math.sin(a)))
    assert torch.isclose(p[3], 1.5 * (x[0, 0, 3] * math.cos(a) + x[0, 0, 2] * math.sin(a)))


def test_plain_window_sink_and_convolution():
    vis = pg.seen_mask(9, 3)
    for i in range(9):
        assert vis[i].nonzero().flatten().tolist() == list(range(max(0, i - 2), i + 1))
    assert torch.equal(pg.seen_mask(5, 0), torch.tril(torch.ones(5, 5, dtype=torch.bool)))
    s = torch.tensor([[[0.5, -math.inf], [1.0, 2.0]]], dtype=F64)
    w = pg.sink_softmax(s, torch.tensor([0.7], dtype=F64))
    assert torch.isclose(w[0, 0, 0], torch.tensor(math.exp(0.5) / (math.exp(0.5) + math.exp(0.7)), dtype=F64)) and w[0, 0, 1] == 0
    assert torch.isclose(w[0, 1, 1], torch.tensor(math.exp(2.0) / (math.exp(1.0) + math.exp(2.0) + math.exp(0.7)), dtype=F64))
    g = torch.Generator().manual_seed(2)
    u, taps = torch.randn(6, 3, generator=g, dtype=F64), torch.randn(3, 4, generator=g, dtype=F64)
    y = pg.causal_conv(u, taps)
    for i in range(6):
        assert torch.allclose(y[i], sum(taps[:, 3 - d] * u[i - d] for d in range(4) if i - d >= 0))
    assert torch.allclose(pg.causal_conv(u[:2], taps), y[:2])                  # fewer rows than taps
    assert abs(float(pg.gelu_tanh(torch.tensor(1.0, dtype=F64))) - 0.8411919906082768) < 1e-12


def test_plain_attention_key_by_key():
    """Both mixers written out head by head and key by key: values are turned by their own position and the sum is turned
    back by the row's, so a key at distance d adds its value turned by -d."""
    g = torch.Generator().manual_seed(3)
    T, W = 6, 9
    m = {"heads": 4, "kv_heads": 2, "dim": 5, "vdim": 4, "conv": 2, "scale": 0.5, "rot": {"dims": 2, "base": 20.0}}
    t = {}
    for n, ch in (("q", 20), ("k", 10), ("v", 8)):
        t.update({n: torch.randn(ch, W, generator=g), n + ".b": torch.randn(ch, generator=g), n + ".conv": torch.randn(ch, 2, generator=g)})
    t.update({"sink": torch.randn(4, generator=g), "o": torch.randn(W, 16, generator=g), "o.b": torch.randn(W, generator=g)})
    t = {k: v.double() for k, v in t.items()}
    h = torch.randn(T, W, generator=g, dtype=F64)
    got = pg.attention(h, t, "", m, torch.arange(T))
    u = {n: h @ t[n].T + t[n + ".b"] for n in "qkv"}
    c = {n: torch.stack([u[n][i] * t[n + ".conv"][:, 1] + (u[n][i - 1] * t[n + ".conv"][:, 0] if i else 0) for i in range(T)]) for n in "qkv"}
    f, fv = pg.frequencies(2, 20.0), pg.frequencies(4, 20.0)
    out = torch.zeros(T, 4, 4, dtype=F64)
    for i in range(T):
        for hd in range(4):
            kv = hd // 2
            e = []
            for j in range(i + 1):
                q = pg.rotate_pairs(c["q"][i].view(4, 5)[None, hd:hd + 1], torch.tensor([i]), 2, f)
                k = pg.rotate_pairs(c["k"][j].view(2, 5)[None, kv:kv + 1], torch.tensor([j]), 2, f)
                e.append(math.exp(float((q * k).sum()) * 0.5))
            z = sum(e) + math.exp(float(t["sink"][hd]))
            for j in range(i + 1):
                out[i, hd] += e[j] / z * pg.rotate_pairs(c["v"][j].view(2, 4)[None, kv:kv + 1], torch.tensor([j - i]), 4, fv)[0, 0]
    assert torch.allclose(got, out.reshape(T, 16) @ t["o"].T + t["o.b"], atol=1e-11)

    m = {"heads": 2, "dim": 3, "rot_dim": 4, "vdim": 2, "kv_rank": 5, "q_rank": 6, "scale": 0.4, "mask": {"size": 3},
         "rot": {"dims": 4, "base": 10.0, "scaling": {"factor": 2.0, "original": 20, "fast": 2.0, "slow": 1.0}}}
    t = {"dq": (6, W), "dq.norm": (6,), "uq": (14, 6), "dkv": (9, W), "dkv.norm": (5,), "uk": (6, 5), "uv": (4, 5), "sink": (2,),
         "g": (4, W), "o": (W, 4)}
    t = {k: torch.randn(s, generator=g, dtype=F64) for k, s in t.items()}
    got = pg.latent_attention(h, t, "", m, 1e-5, torch.arange(T))
    fr, factor = pg.slowed(4, 10.0, m["rot"]["scaling"])
    rms = lambda x: x / math.sqrt(float((x * x).mean()) + 1e-5)
    out = torch.zeros(T, 4, dtype=F64)
    for i in range(T):
        q = (t["uq"] @ (rms(t["dq"] @ h[i]) * t["dq.norm"])).view(2, 7)
        gate = torch.sigmoid(t["g"] @ h[i])
        for hd in range(2):
            e, v = [], []
            for j in range(max(0, i - 2), i + 1):
                a = t["dkv"] @ h[j]
                cc = rms(a[:5]) * t["dkv.norm"]
                qr = pg.rotate_half(q[None, hd:hd + 1, 3:], torch.tensor([i]), 4, fr, factor)
                kr = pg.rotate_half(a[None, None, 5:], torch.tensor([j]), 4, fr, factor)
                e.append(math.exp(0.4 * float(q[hd, :3] @ (t["uk"] @ cc).view(2, 3)[hd] + (qr * kr).sum())))
                v.append((t["uv"] @ cc).view(2, 2)[hd])
            z = sum(e) + math.exp(float(t["sink"][hd]))
            out[i, 2 * hd:2 * hd + 2] = sum(x / z * y for x, y in zip(e, v)) * gate[2 * hd:2 * hd + 2]
    assert torch.allclose(got, out @ t["o"].T, atol=1e-11)


# ---- the engine on the stand-ins against the plain implementation ---------------------------------------------------

@pytest.mark.parametrize("name", list(GM.CONFIGS))
def test_schedules_on_the_stand_in(name):
    cfg, w, w64 = model(name)
    reqs = {f"r{i}": H.random_ids(cfg["vocab"], n, 40 + i) for i, n in enumerate([37, 1, 58, 23, 70])}
    eng = engine_for(cfg, w)
    for steps in (H.whole_trace(reqs), H.tail_decode_trace(reqs, tail=12), H.portions_trace(reqs, seed=3)):
        got = GM.run_trace(eng, steps)
        assert len(got) == sum(len(v) for v in reqs.values())
        worst = GM.worst_error(name, cfg, w64, reqs, got)
        assert worst[0] <= TOL32, worst
        assert eng.cache.n_live == 0
        eng.cache.check()
    # several requests at a time with pages for the live ones only: pages and state slots are used again
    steps, peak = H.mixed_trace(reqs, max_live=3, seed=4)
    eng = engine_for(cfg, w, max_requests=3, max_tokens=peak, graphs=True)
    worst = GM.worst_error(name, cfg, w64, reqs, GM.run_trace(eng, steps))
    assert worst[0] <= TOL32, worst
    eng.cache.check()


def test_the_streams_after_every_pass():
    """Beside the logits: the sum of the streams after every layer run (a layer that is passed again counts each time)."""
    cfg, w, w64 = model("A")
    ids = H.random_ids(cfg["vocab"], 25, 3)
    want = []
    pg.forward(cfg, w64, ids, want)
    eng = engine_for(cfg, w)
    got = []
    for layer in {id(l): l for l in eng.model.layers}.values():
        inner = layer.forward
        layer.forward = lambda x, ctx, inner=inner: (lambda out: (got.append(out.full.sum(1).double()), out)[1])(inner(x, ctx))
    eng.step([("a", ids, [0])])
    assert len(got) == len(want) == 6
    for a, b in zip(got, want):
        assert (a - b).abs().max() <= 1e-4 * b.abs().max()


def test_a_used_state_slot_starts_from_zero():
    cfg, w, w64 = model("A")
    eng = engine_for(cfg, w, max_requests=1)
    ids_a, ids_b = H.random_ids(cfg["vocab"], 30, 1), H.random_ids(cfg["vocab"], 9, 2)
    GM.run_trace(eng, H.whole_trace({"a": ids_a}))
    assert all(t[0].abs().max() > 0 for t in eng.cache.states.values())     # the first request left its state in the only slot
    got = GM.run_trace(eng, H.portions_trace({"b": ids_b}, sizes=(2, 3)))
    assert GM.worst_error("A", cfg, w64, {"b": ids_b}, got)[0] <= TOL32


def needle_case(name, at, distance, window=None, first=0, seed=60):
    """A sequence in which the probe token, `distance` after the needle at `at`, looks for it in the first layer (the
    configuration's layer `first` moved there; its window set to `window` if given); and how far the probe's logits move
    when the needle is replaced."""
    cfg = copy.deepcopy(GM.CONFIGS[name])
    cfg["layers"].insert(0, cfg["layers"].pop(first))
    if window is not None:
        cfg["layers"][0]["mixer"]["mask"] = {"size": window}
    needle, probe = 3, 7
    w = GM.sharpen(cfg, GM.random_weights(cfg, 5), needle, probe, distance)
    w64 = GM.as_f64(w)
    ids = [t if t not in (needle, probe) else 11 for t in H.random_ids(cfg["vocab"], at + distance + 4, seed + at)]
    ids[at], ids[at + distance] = needle, probe
    without = list(ids)
    without[at] = 11
    key = (name, "sharp", first, window, distance)
    want = GM.plain_logits(key, cfg, w64, ids)[at + distance]
    moved = GM.relative_error(pg.forward(cfg, w64, without)[at + distance], want)
    return key, cfg, w, w64, ids, moved


def run_three_ways(key, cfg, w, w64, ids, tail=6):
    eng = engine_for(cfg, w)
    for steps in (H.whole_trace({"s": ids}), H.tail_decode_trace({"s": ids}, tail=tail),
                  H.portions_trace({"s": ids}, sizes=(5, 2, 11))):
        got = GM.run_trace(eng, steps)
        worst = GM.worst_error(key, cfg, w64, {"s": ids}, got)
        assert worst[0] <= TOL32, worst


@pytest.mark.parametrize("name,distance,first,window", [("A", 1, 0, None), ("C", 240, 0, None), ("C", 150, 1, 200), ("B", 60, 0, None)])
def test_a_token_that_stands_out(name, distance, first, window):
    """The probe looks for a needle right before it or hundreds of tokens back, with the needle on both sides of a page's
    border; whole, decoded alone and in portions."""
    for at in (15, 16):
        key, cfg, w, w64, ids, moved = needle_case(name, at, distance, window, first)
        assert moved >= 0.01, moved              # losing that one key would show
        run_three_ways(key, cfg, w, w64, ids)


@pytest.mark.parametrize("window", [2, 21, 32])
def test_keys_just_inside_and_just_outside_a_window(window):
    """Windows that end inside a page and at a page's border: the needle is the farthest key the probe sees, and the next
    one that it does not; in prompts, in portions, and decoded past the edge (pages behind the window have gone back)."""
    for at in (39, 40, 47):
        for distance, seen in ((window - 1, True), (window, False)):
            key, cfg, w, w64, ids, moved = needle_case("A", at, distance, window)
            if seen:
                assert moved >= 0.01, (at, distance, moved)
            else:
                without = list(ids)
                without[at] = 11
                rows = []
                for seq in (ids, without):
                    h = pg.rms_norm(w64["embed"][torch.tensor(seq)] * w64["l0.hc1.in"].sum(), w64["l0.norm1"], cfg["norm"]["eps"])
                    rows.append(pg.latent_attention(h, w64, "l0.mix.", cfg["layers"][0]["mixer"], cfg["norm"]["eps"], torch.arange(len(seq)))[at + distance])
                assert torch.equal(rows[0], rows[1])
            run_three_ways(key, cfg, w, w64, ids, tail=window + 3)


def test_the_first_tokens_and_one_token_alone():
    for name in GM.CONFIGS:
        cfg, w, w64 = model(name, seed=7)
        eng = engine_for(cfg, w)
        reqs = {"one": H.random_ids(cfg["vocab"], 1, 1), "two": H.random_ids(cfg["vocab"], 2, 2), "five": H.random_ids(cfg["vocab"], 5, 3)}
        for steps in (H.whole_trace(reqs), H.tail_decode_trace(reqs, tail=4)):
            got = GM.run_trace(eng, steps)
            assert GM.worst_error((name, 7), cfg, w64, reqs, got)[0] <= TOL32


def test_long_decoding_of_unequal_requests():
    """Three requests of unequal lengths decode 90 tokens together, over page borders and window edges, each against
    itself alone."""
    cfg, w, w64 = model("A", seed=6)
    reqs = {f"r{i}": H.random_ids(cfg["vocab"], n, 90 + i) for i, n in enumerate([100, 131, 93])}
    eng = engine_for(cfg, w, max_requests=3, graphs=True)
    steps = [{"step": 0, "entries": [{"id": r, "tokens": ids[:len(ids) - 90], "want": [0]} for r, ids in reqs.items()], "end": []}]
    for t in range(90):
        steps.append({"step": t + 1, "entries": [{"id": r, "tokens": [ids[len(ids) - 90 + t]], "want": [0]} for r, ids in reqs.items()],
                      "end": list(reqs) if t == 89 else []})
    got = GM.run_trace(eng, steps)
    assert GM.worst_error(("A", 6), cfg, w64, reqs, got)[0] <= TOL32
    eng.cache.check()


def test_what_the_design_fixes_shows_in_the_logits():
    """Leaving a mechanism out, or doing it in the other order or the other layout, moves the plain logits by far more than
    the engine's tolerance: the schedules above would catch any of them."""
    cfg, w, w64 = model("A")
    ids = H.random_ids(cfg["vocab"], 60, 9)
    want = GM.plain_logits("A", cfg, w64, ids)
    wrong = {
        "sink_softmax": lambda s, sink: torch.softmax(s, dim=-1),
        "token_shift": lambda h, a: h,
        "causal_conv": lambda x, taps: x * taps[:, -1],
        "write_streams": lambda X, mix, out, y: torch.einsum("ts,slw->tlw", mix, X) + out.view(-1, 1, 1) * y,
        "read_streams": lambda X, weights: X.mean(0),
        "rotate_half": pg.rotate_pairs,
        "rotate_pairs": lambda x, p, dims, f, factor=1.0: pg.rotate_half(x, p, dims, f, factor),
        "slowed": lambda dims, base, sc: (pg.frequencies(dims, base), 1.0),
        "seen_mask": lambda T, window: (lambda d: (d >= 0) & (d <= window) if window else d >= 0)(
            torch.arange(T).view(-1, 1) - torch.arange(T).view(1, -1)),
    }
    for name, fn in wrong.items():
        keep = getattr(pg, name)
        half = pg.rotate_half
        try:
            setattr(pg, name, fn if name != "rotate_pairs" else lambda x, p, dims, f, factor=1.0: half(x, p, dims, f, factor))
            moved = max(GM.relative_error(pg.forward(cfg, w64, ids)[t], want[t]) for t in (20, 59))
        finally:
            setattr(pg, name, keep)
        assert moved > 100 * TOL32, (name, moved)
    # values that are turned but not turned back
    keep = pg.rotate_pairs
    try:
        pg.rotate_pairs = lambda x, p, dims, f, factor=1.0: x if int(p.min()) < 0 else keep(x, p, dims, f, factor)
        assert GM.relative_error(pg.forward(cfg, w64, ids)[59], want[59]) > 100 * TOL32
    finally:
        pg.rotate_pairs = keep


def test_greedy_generation_through_the_scheduler():
    for name in ("A", "B"):
        cfg, w, w64 = model(name, seed=8)
        prompts = [H.random_ids(cfg["vocab"], n, 80 + i) for i, n in enumerate((13, 1, 30, 6))]
        want = [pg.greedy_generate(cfg, w64, p, 7) for p in prompts]
        eng = engine_for(cfg, w, max_requests=2, max_tokens=160, graphs=True)
        out, s = generate(eng, prompts, max_new_tokens=7, temperature=0.0, max_batch=2, token_budget=11,
                          return_scheduler=True)
        assert out == want
        assert s.peak_running == 2 and eng.cache.n_live == 0
        eng.cache.check()


def test_the_named_size_runs_with_random_weights(tmp_path):
    from tiny_inference_server_amd.__main__ import preset_names, size_config
    from tiny_inference_server_amd.weights import write_random_model
    assert "gosavik-small" in preset_names()
    cfg = size_config("gosavik-small")
    folder = write_random_model(cfg, 3, str(tmp_path / "m"))
    assert load_config(folder).to_dict() == cfg.to_dict()
    eng = Engine(folder, dtype="float32", max_tokens=64, max_requests=2, ops=TorchOps())
    out = eng.step([("a", [5, 9, 1, 300], [3]), ("b", [7], [0])]).logits
    assert out.shape == (2, cfg.vocab) and torch.isfinite(out).all()
