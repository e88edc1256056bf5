"""Lunulix on the framework's CPU semantics against the plain oracle:
mechanisms, schedules, cache and slots, scheduler, loading, command line."""

import io
import json
import math
import os
import subprocess
import sys

import lunulix_cases as C
import lunulix_oracle as O
import numpy as np
import pytest
import torch

from quickstart_streaming_agents_amd.models import build_model, load_model
from quickstart_streaming_agents_amd.models.kv_cache import HybridCache
from quickstart_streaming_agents_amd.models.layers import (RopeTable,
                                                           StepPlan,
                                                           TokenSide)
from quickstart_streaming_agents_amd.models.lunulix import LunulixConfig
from quickstart_streaming_agents_amd.models.weights import write_safetensors
from quickstart_streaming_agents_amd.ops import dispatch as D

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
F32 = torch.float32


def gen(seed):
    return torch.Generator().manual_seed(seed)


@pytest.fixture(scope="module")
def cases():
    return {k: C.Case(k) for k in C.CONFIGS}


# ---- mechanisms alone -------------------------------------------------------

def test_residual_norm_with_post_norm():
    g = gen(1)
    T, W, V = 5, 52, 9
    res, y = torch.randn(T, W, generator=g), torch.randn(T, W, generator=g)
    table, ids = torch.randn(V, W, generator=g), torch.tensor([3, 0, 8, 8, 1])
    w, post = torch.randn(W, generator=g), torch.randn(W, generator=g)
    for init in (False, True):
        r = res.clone()
        out = D.residual_norm(r, y, w, None, 1e-3, table=table, ids=ids,
                              init=init, layer=False, post=post, tscale=2.5)
        x = (0 if init else res.double()) + 2.5 * table.double()[ids] + \
            O.rms(y.double(), 1e-3, post.double())
        assert torch.allclose(r.double(), x, atol=1e-5)
        assert torch.allclose(out.double(), O.rms(x, 1e-3, w.double()),
                              atol=1e-5)
    r = res.clone()
    out = D.residual_norm(r, y, None, None, 1e-3, post=post)
    assert torch.equal(out, r) and out.data_ptr() != r.data_ptr()


def test_gelu_unit_and_token_side():
    g = gen(2)
    x = torch.randn(7, 24, generator=g) * 3
    assert torch.allclose(
        D.glu(x[:, :12], x[:, 12:], "gelu").double(),
        O.gelu_tanh(x[:, :12].double()) * x[:, 12:].double(), atol=1e-5)
    gate, proj = torch.randn(5, 20, generator=g), torch.randn(20, 5,
                                                              generator=g)
    table = torch.randn(11, 15, generator=g)
    ids = torch.tensor([4, 0, 10, 4])
    h = torch.randn(4, 20, generator=g)
    for layer in range(3):
        got = TokenSide(gate, proj, table, layer)(h, ids)
        e = table[ids][:, layer * 5:layer * 5 + 5].double()
        want = (O.gelu_tanh(h.double() @ gate.double().T) * e) \
            @ proj.double().T
        assert torch.allclose(got.double(), want, atol=1e-4)


@pytest.mark.parametrize("dims,base,scaling", [
    (16, 1e4, None), (64, 1e6, C.STRETCH), (20, 1e3, {
        "factor": 2.5, "low": 0.5, "high": 9.0, "original": 80}),
    (0, 1.0, None)])
def test_rotation_frequencies(dims, base, scaling):
    t = RopeTable(dims, base, "cpu", scaling)
    t.ensure(300)
    want = O.frequencies(dims, base, scaling)
    assert t.cos.shape == (512, dims // 2)
    for i, f in enumerate(want):
        assert math.isclose(float(t.freq[i]), f, rel_tol=1e-12)
        assert abs(float(t.cos[299, i]) - math.cos(299 * f)) < 1e-6
        assert abs(float(t.sin[299, i]) - math.sin(299 * f)) < 1e-6
    if scaling:      # all three regimes are there
        plain = O.frequencies(dims, base)
        ratio = {round(a / b, 6) for a, b in zip(want, plain)}
        assert 1.0 in ratio and round(1 / scaling["factor"], 6) in ratio
        assert len(ratio) > 2


def _portion_tensors(cuts):
    """Plan arrays of one sequence's portions run one after the other."""
    at = 0
    for n in cuts:
        i32 = lambda *v: torch.tensor(v, dtype=torch.int32)
        t0 = list(range(0, n, StepPlan.CONV_ROWS))
        if n == 1:
            yield at, n, (None, None, None, i32(at + 1), None, i32(2))
        else:
            yield at, n, (i32(*[0] * len(t0)), i32(*t0), i32(0), i32(at),
                          i32(n), i32(2))
        at += n


@pytest.mark.parametrize("taps", [1, 2, 4, 7])
def test_short_convolution(taps):
    g = gen(taps)
    x, w = torch.randn(60, 10, generator=g), torch.randn(10, taps,
                                                         generator=g)
    b = torch.randn(10, generator=g)
    want = O.silu(O.short_conv(x.double(), w.double(), b.double()))
    tails = torch.full((3, taps - 1, 10), float("nan"))
    for at, n, conv in _portion_tensors([1, 2, 3, 1, 1, 40, 2, 10]):
        got = D.conv_silu(x[at:at + n], w.t().contiguous(), b, tails, *conv)
        assert torch.allclose(got.double(), want[at:at + n], atol=1e-5)


def _mixer_alone(config, mixer_fn, h):
    case = C.Case(None, config=config)
    kv = case.model.new_kv_cache(4, 2)
    kv.allocate(0, h.shape[0])
    plan = StepPlan.build([(torch.zeros(h.shape[0], dtype=torch.int64), 0,
                            0)], kv)
    return case, kv, plan


@pytest.mark.parametrize("H,G,dim,vdim,rot", [
    (4, 4, 10, 6, 4), (6, 2, 8, 12, 8), (3, 1, 6, 6, 0)])
def test_attention_branch(H, G, dim, vdim, rot):
    m = C.left(H, G, dim, vdim, 3, rot, 0.9, 300.0, C.STRETCH)
    cfg = C.model(50, 24, 4, C.par(m, C.right(1, 4, 4, 1, 2, 1)))
    h = torch.randn(140, 24, generator=gen(3))
    case, kv, plan = _mixer_alone(cfg, None, h)
    mix = case.model.layers[0].mixer
    x = mix.proj(h)
    y = torch.zeros(140, H * vdim)
    mix.left(x[:, :mix.at], plan, kv, 0, kv.tails[0][0], y)
    W = O.sub(case.weights, "l0.mix.left.")
    want = O.attention_branch(h.double(), W, m)
    got = y.double() / 0.8 @ W["o"].T
    assert torch.allclose(got, want, atol=1e-4)


@pytest.mark.parametrize("H,P,N,G,parts", [
    (4, 5, 6, 2, 1), (3, 8, 4, 1, 6), (2, 6, 8, 2, 2)])
def test_state_space_branch(H, P, N, G, parts):
    m = C.right(H, P, N, G, 4, parts)
    cfg = C.model(50, 24, 4, C.par(C.left(1, 1, 4, 4, 2, 2, 1.0), m),
                  eps=1e-4)
    h = torch.randn(70, 24, generator=gen(4))
    case, kv, plan = _mixer_alone(cfg, None, h)
    mix = case.model.layers[0].mixer
    x = mix.proj(h)
    y = torch.zeros(70, H * P)
    mix.right(x[:, mix.at:], plan, kv, 0, kv.tails[0][1], y)
    W = O.sub(case.weights, "l0.mix.right.")
    want = O.ssd_branch(h.double(), W, m, 1e-4)
    assert torch.allclose(y.double() / 1.3 @ W["o"].T, want, atol=1e-4)
    whole = mix(h, plan, kv, 0).double()
    Wm = O.sub(case.weights, "l0.mix.")
    assert torch.allclose(whole, O.parallel_mixer(
        h.double(), Wm, cfg["layers"][0]["mixer"], 1e-4), atol=1e-4)


def test_residual_after_every_layer(cases):
    for case in cases.values():
        toks = case.tokens(21)
        kv = case.model.new_kv_cache(2, 1)
        kv.allocate(0, 21)
        trail = []
        case.model.forward_prefill_batch([(torch.tensor(toks), 0, 0)], kv,
                                         trail=trail)
        want = O.forward(case.raw, case.weights, toks)[1]
        assert len(trail) == len(want)
        for a, b in zip(trail, want):
            assert torch.allclose(a.double(), b, atol=2e-4)


# ---- the checks see a planted mistake (made in the oracle) ------------------

def _swap_scales(cfg):
    for L in cfg["layers"]:
        m = L["mixer"]
        m["left_scale"], m["right_scale"] = m["right_scale"], m["left_scale"]


def _all(cfg, key, value, side="left"):
    for L in cfg["layers"]:
        L["mixer"][side][key] = value


CONFIG_MISTAKES = {
    "scales swapped": _swap_scales,
    "frequencies unscaled": lambda c: [
        L["mixer"]["left"]["rot"].update(scaling=None) for L in c["layers"]],
    "fewer dims rotated": lambda c: [
        L["mixer"]["left"]["rot"].update(dims=L["mixer"]["left"]["rot"]
                                         ["dims"] // 2) for L in c["layers"]],
    "norm in one part": lambda c: _all(c, "norm_groups", 1, "right"),
    "embedding unscaled": lambda c: c["embedding"].update(scale=1.0),
    "no feed-forward": lambda c: c["layers"][1].update(mlp=None),
}
WEIGHT_MISTAKES = {
    "no sink": ("sink", lambda w: torch.full_like(w, -1e4)),
    "convolution reversed": ("conv", lambda w: w.flip(1)),
    "convolution one late": ("conv", lambda w: w.roll(1, 1)),
    "no convolution bias": ("conv.b", torch.zeros_like),
    "no step bias": ("dt_bias", torch.zeros_like),
    "no skip": ("right.D", torch.zeros_like),
    "one decay": ("A_log", torch.zeros_like),
    "no norm weight": ("right.norm", torch.ones_like),
    "mixer's end norm": ("norm1b", torch.ones_like),
    "feed-forward's end norm": ("norm2b", torch.ones_like),
    "no side input": ("side.norm", torch.zeros_like),
    "next layer's side input": ("side.embed", lambda w: w.roll(56, 1)),
}
FUNCTION_MISTAKES = {
    "gelu by erf": ("gelu_tanh", lambda z: 0.5 * z * (
        1 + torch.erf(z / math.sqrt(2)))),
    "softplus clamped": ("softplus", lambda z: torch.log1p(
        torch.exp(z)).clamp(max=0.5)),
    "gate after the norm": ("gated_group_norm", lambda y, z, w, parts, eps:
                            O.rms(y.view(y.shape[0], parts, -1), eps)
                            .reshape(y.shape) * w * O.silu(z)),
}


@pytest.mark.parametrize("mistake", [*CONFIG_MISTAKES, *WEIGHT_MISTAKES,
                                     *FUNCTION_MISTAKES])
def test_planted_mistakes_show(cases, monkeypatch, mistake):
    case = cases["tiles"]
    toks = case.tokens(130, seed=4)
    right = case.oracle(toks)
    cfg, weights = json.loads(json.dumps(case.raw)), dict(case.weights)
    if mistake in CONFIG_MISTAKES:
        CONFIG_MISTAKES[mistake](cfg)
    elif mistake in WEIGHT_MISTAKES:
        end, fn = WEIGHT_MISTAKES[mistake]
        hits = [k for k in weights if k.endswith(end)]
        assert hits
        weights.update({k: fn(weights[k]) for k in hits})
    else:
        name, fn = FUNCTION_MISTAKES[mistake]
        monkeypatch.setattr(O, name, fn)
    wrong = O.forward(cfg, weights, toks)[0]
    assert float(C.row_errors(wrong.float(), right).max()) > \
        2.5 * C.TOL[F32] * (1 if mistake == "gelu by erf" else 10)


# ---- schedules --------------------------------------------------------------

@pytest.mark.parametrize("cuts", C.CUTS)
@pytest.mark.parametrize("name", C.CONFIGS)
def test_cuts(cases, name, cuts):
    C.scenario_cuts(cases[name], 150, cuts)


@pytest.mark.parametrize("name", C.CONFIGS)
def test_mixed_batches(cases, name):
    C.scenario_mixed(cases[name])


@pytest.mark.parametrize("name", ["odd", "tiles"])
def test_slot_and_page_reuse(cases, name):
    C.scenario_reuse(cases[name])


@pytest.mark.parametrize("spot,n", [(0, 200), (63, 150), (64, 200)])
@pytest.mark.parametrize("cuts", [
    lambda n: [n], lambda n: [n - 12] + [1] * 12,
    lambda n: C.portions(n, [2, 37])], ids=["prompt", "decoded", "portions"])
def test_far_keys(spot, n, cuts):
    C.scenario_far_key(spot, n, "cpu", F32, cuts)


def test_long_decoding(cases):
    C.scenario_cuts(cases["ones"], 400, "decoded tail")


# ---- scheduler --------------------------------------------------------------

@pytest.mark.parametrize("name", ["odd", "tiles", "ones"])
@pytest.mark.parametrize("chunk", [None, 24])
def test_generation(cases, name, chunk):
    C.scenario_generate(cases[name], chunk_tokens=chunk)


def test_conversations_reuse_the_snapshot(cases):
    C.scenario_conversation(cases["odd"])


def test_snapshot_keeps_the_convolutions_inputs():
    kv = HybridCache(8, 3, [], [(1, 2, 2)], device="cpu", dtype=F32,
                     kv_shapes=[(2, 4, 6)], tail_shapes=[((2, 5), (3, 7))])
    assert kv.keys[0].shape == (8, 2, 64, 4)
    assert kv.values[0].shape == (8, 2, 64, 6)
    kv.allocate(1, 10)
    for t in (kv.states[0], *kv.tails[0]):
        t[kv.slot(1)] = 5.0
    kv.snapshot(1)
    for t in (kv.states[0], *kv.tails[0]):
        t[kv.slot(1)] = 7.0
    kv.extend(1, 20)
    kv.truncate(1, 10)
    for t in (kv.states[0], *kv.tails[0]):
        assert float(t[kv.slot(1)].min()) == 5.0


# ---- loading, registry, command line ----------------------------------------

@pytest.fixture(scope="module")
def folder(tmp_path_factory):
    case = C.Case("odd", seed=5)
    d = tmp_path_factory.mktemp("model")
    (d / "config.json").write_text(json.dumps(case.raw))
    write_safetensors(str(d / "model.safetensors"), case.weights)
    return case, str(d)


def test_load_by_architecture(folder):
    case, d = folder
    assert case.cfg.to_dict() == case.raw
    for m in (load_model(d, device="cpu"), build_model(d, device="cpu")):
        assert m.cfg.to_dict() == case.cfg.to_dict()
        assert torch.equal(m.embed, case.model.embed)


def test_wrong_shapes_are_refused(folder, tmp_path):
    case, _ = folder
    (tmp_path / "config.json").write_text(json.dumps(case.raw))
    bad = dict(case.weights)
    bad["l0.mix.left.k"] = bad["l0.mix.left.k"][:-1].contiguous()
    write_safetensors(str(tmp_path / "model.safetensors"), bad)
    with pytest.raises(ValueError, match="l0.mix.left.k"):
        load_model(str(tmp_path), device="cpu")
    del bad["l0.mix.left.k"]
    write_safetensors(str(tmp_path / "model.safetensors"), bad)
    with pytest.raises(KeyError, match="l0.mix.left.k"):
        load_model(str(tmp_path), device="cpu")


def test_unknown_parts_are_refused():
    cfg = C.model(50, 24, 4, dict(C.CONFIGS["odd"]["layers"][0],
                                  type="spiral"))
    with pytest.raises(ValueError, match="spiral"):
        LunulixConfig.from_dict(cfg)
    cfg = json.loads(json.dumps(C.CONFIGS["odd"]))
    cfg["layers"][0]["mlp"]["kind"] = "sparse"
    with pytest.raises(ValueError, match="sparse"):
        LunulixConfig.from_dict(cfg)


def test_presets():
    m = build_model("tiny-lunulix", device="cpu", seed=1)
    from quickstart_streaming_agents_amd.models.serve import Engine
    outs = Engine(m, max_batch=2, max_seq_len=256).generate_batch(
        [[1, 2, 3], [9] * 70], [5, 5])
    assert [len(o) for o in outs] == [5, 5]
    for name in ("lunulix-1b", "lunulix-8b"):
        assert LunulixConfig.preset(name).layers


def test_replay_protocol(folder, tmp_path, monkeypatch, capsys):
    from quickstart_streaming_agents_amd.models import replay
    case, d = folder
    a, b = case.tokens(70, 1), case.tokens(9, 2)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:66], "want": [0, 65]},
                                {"id": "b", "tokens": b[:1], "want": []}],
         "end": []},
        {"step": 1, "entries": [{"id": "b", "tokens": b[1:2], "want": []}],
         "end": []},
        {"step": 2, "entries": [{"id": "b", "tokens": b[2:], "want": [6]},
                                {"id": "a", "tokens": a[66:67],
                                 "want": [0]}], "end": ["b"]},
        {"step": 3, "entries": [{"id": "a", "tokens": a[67:68],
                                 "want": [0]}], "end": ["a"]}]
    monkeypatch.setattr("sys.stdin", io.StringIO(
        "\n".join(json.dumps(s) for s in steps) + "\n"))
    assert replay.main(["--model", d, "--dtype", "float32", "--out",
                        str(tmp_path), "--max-tokens", "192",
                        "--device", "cpu"]) == 0
    said = capsys.readouterr().out.split("\n")
    assert said[:4] == [f"done {i}" for i in range(4)]
    assert not (tmp_path / "1.f32").exists()
    A, B = case.oracle(a[:68]), case.oracle(b)
    for step, want in ((0, A[[0, 65]]), (2, torch.stack([B[8], A[66]])),
                       (3, A[67:68])):
        got = torch.from_numpy(np.fromfile(tmp_path / f"{step}.f32", "<f4"))
        C.check(case, got.view(len(want), -1), want, f"step {step}")


def test_generate_command(folder):
    case, d = folder
    r = subprocess.run(
        [sys.executable, "-m", "quickstart_streaming_agents_amd", "generate",
         "--model", d, "--tokens", "3,1,4,1,5", "--max-new", "6",
         "--device", "cpu"], cwd=ROOT, capture_output=True, text=True)
    assert r.returncode == 0, r.stderr
    out = json.loads(r.stdout.strip().splitlines()[-1])
    assert len(out["tokens"]) == 6
    C.greedy_check(case, [3, 1, 4, 1, 5], out["tokens"])


# ---- tensor parallelism -----------------------------------------------------

TP_CONFIG = C.model(
    128, 48, 8, C.par(C.left(4, 2, 8, 12, 3, 8, 0.4),
                      C.right(6, 6, 8, 2, 4, 4), 64),
    C.par(C.left(2, 2, 10, 8, 2, 4, 0.4), C.right(2, 8, 5, 2, 3, 2)))


def _tp_worker(rank, world):
    import torch.distributed as dist

    from quickstart_streaming_agents_amd.models.lunulix import LunulixModel
    from quickstart_streaming_agents_amd.models.serve import Engine
    dist.init_process_group("gloo")
    cfg = LunulixConfig.from_dict(TP_CONFIG)
    m = LunulixModel(cfg, device="cpu", dtype=F32,
                     weights=C.make_weights(cfg), tp_rank=rank,
                     tp_size=world)
    outs = Engine(m, max_batch=2, max_seq_len=128).generate_batch(
        [[1, 5, 9, 13] * 8, [2, 4, 6]], [9, 9])
    dist.destroy_process_group()
    return outs


@pytest.mark.timeout(300)
def test_tp2_matches_tp1():
    from test_parallel import spawn_world
    case = C.Case(None, config=TP_CONFIG)
    got = spawn_world(_tp_worker, world=2)
    assert got[0] == got[1]
    for p, o in zip([[1, 5, 9, 13] * 8, [2, 4, 6]], got[0]):
        C.greedy_check(case, p, o)
