"""Lunulix on the GPU: every kernel against plain f64 references of the same
mechanism, then the model through the framework's step function, cache,
scheduler and graph against the oracle, in f32 and bf16."""

import lunulix_cases as C
import lunulix_oracle as O
import pytest
import torch

from quickstart_streaming_agents_amd.models.layers import RopeTable, StepPlan
from quickstart_streaming_agents_amd.ops import dispatch as D

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
F32, BF = torch.float32, torch.bfloat16
BOTH = pytest.mark.parametrize("dtype", [F32, BF], ids=["f32", "bf16"])


def gen(seed):
    return torch.Generator().manual_seed(seed)


def rnd(g, *shape, dtype=F32, scale=1.0):
    return (torch.randn(*shape, generator=g) * scale).to(dtype)


def i32(*v):
    return torch.tensor(v, dtype=torch.int32, device=DEV)


def close(got, want, dtype):
    """Largest rms error of a row, relative to the rms of everything."""
    got, want = got.double().cpu(), want.double()
    rms = want.pow(2).mean().sqrt().clamp(min=1e-6)
    err = (got - want).pow(2).mean(-1).sqrt().max() / rms
    assert float(err) <= (2e-5 if dtype == F32 else 3e-2), float(err)


# ---- row kernels ------------------------------------------------------------

@BOTH
@pytest.mark.parametrize("W", [33, 100, 256, 4096, 8448])
@pytest.mark.parametrize("layer", [False, True])
def test_residual_norm_with_post_norm(W, layer, dtype):
    g = gen(W)
    T, V = 7, 11
    res, y = rnd(g, T, W), rnd(g, T, W, dtype=dtype)
    table, ids = rnd(g, V, W, dtype=dtype), torch.tensor([0, 10, 3, 3, 1, 9, 2])
    w, post = rnd(g, W, dtype=dtype), rnd(g, W, dtype=dtype)
    p = O.rms(y.double(), 1e-4, post.double())
    for init, full in ((True, True), (False, False)):
        r = res.to(DEV)
        out = D.residual_norm(
            r, y.to(DEV), w.to(DEV), None, 1e-4,
            table=table.to(DEV) if full else None,
            ids=ids.to(DEV) if full else None, init=init, layer=layer,
            post=post.to(DEV), tscale=3.5)
        x = p + (0 if init else res.double())
        if full:
            x = x + 3.5 * table.double()[ids]
        close(r, x, F32)
        c = x - x.mean(-1, keepdim=True) if layer else x
        close(out, O.rms(c, 1e-4, w.double()), dtype)
    # no weight: the stream itself
    r = res.to(DEV)
    out = D.residual_norm(r, y.to(DEV), None, None, 1e-4, post=post.to(DEV))
    close(r, res.double() + p, F32)
    close(out, res.double() + p, dtype)


@BOTH
@pytest.mark.parametrize("cols", [5, 24, 90, 264])
def test_gelu_units(cols, dtype):
    g = gen(1)
    x = rnd(g, 19, 2 * cols, dtype=dtype, scale=3.0)
    d = x.to(DEV)
    want = O.gelu_tanh(x[:, :cols].double())
    close(D.glu(d[:, :cols], d[:, cols:], "gelu"),
          want * x[:, cols:].double(), dtype)
    table = rnd(g, 13, 3 * cols, dtype=dtype)
    ids = torch.randint(0, 13, (19,), generator=g)
    for layer in range(3):
        got = D.glu_table(d[:, :cols], table.to(DEV), ids.to(DEV),
                          layer * cols)
        close(got, want * table[ids].double()[:, layer * cols:
                                              (layer + 1) * cols], dtype)


@BOTH
@pytest.mark.parametrize("parts,n", [(1, 36), (3, 7), (8, 512), (2, 1200),
                                     (5, 260)])
def test_part_norm(parts, n, dtype):
    g = gen(n)
    x, w = rnd(g, 9, parts * n, dtype=dtype), rnd(g, parts * n)
    out = torch.zeros(9, parts * n + 8, dtype=dtype, device=DEV)
    D.part_norm(x.to(DEV), w.to(DEV), out[:, 8:], parts, 1e-3)
    want = O.rms(x.double().view(9, parts, n), 1e-3).reshape(9, -1) * \
        w.double()
    close(out[:, 8:], want, dtype)
    assert not out[:, :8].any()


# ---- short convolutions -----------------------------------------------------

def _steps(lens, at):
    """Plan arrays of a step that brings lens[i] tokens from at[i] on for
    sequence i in slot 4 - i, all portions in one launch."""
    n = torch.tensor(lens)
    off = (n.cumsum(0) - n).tolist()
    item, t0 = [], []
    for i, m in enumerate(lens):
        for t in range(0, m, StepPlan.CONV_ROWS):
            item.append(i)
            t0.append(t)
    slots = [4 - i for i in range(len(lens))]
    return i32(*item), i32(*t0), i32(*off), i32(*at), i32(*lens), i32(*slots)


SCHEDULE = [[2, 17, 1, 40], [1, 1, 3, 2], [1, 1, 1, 1], [30, 2, 16, 1],
            [1, 1, 1, 1]]


@BOTH
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 7])
@pytest.mark.parametrize("H,G,Dm,E,rot", [
    (3, 3, 13, 7, 6), (4, 2, 16, 24, 8), (6, 1, 32, 12, 32), (2, 1, 20, 8, 0)])
def test_conv_qkv(H, G, Dm, E, rot, taps, dtype):
    """Four sequences in steps of portions and single tokens: filters, turned
    q and k, pages, tails that start as garbage."""
    g = gen(taps * 100 + H)
    c = (H + G) * Dm + G * E
    total = [sum(s[i] for s in SCHEDULE) for i in range(4)]
    u = [rnd(g, t, c, dtype=dtype) for t in total]
    w = rnd(g, c, taps, dtype=BF)
    rope = RopeTable(rot, 500.0, DEV, C.STRETCH)
    rope.ensure(300)
    want = []
    for x in u:
        y = O.short_conv(x.double(), w.double())
        pos = torch.arange(len(x)).double()
        qk = O.rotate(y[:, :(H + G) * Dm].view(-1, H + G, Dm), pos, rot,
                      500.0, C.STRETCH)
        want.append((qk[:, :H].reshape(-1, H * Dm), qk[:, H:],
                     y[:, (H + G) * Dm:].view(-1, G, E)))
    tails = torch.full((6, taps - 1, c), float("nan"), dtype=dtype,
                       device=DEV)
    kc = torch.zeros(9, G, 64, Dm, dtype=dtype, device=DEV)
    vc = torch.zeros(9, G, 64, E, dtype=dtype, device=DEV)
    pages = [[7, 3], [1, 8], [0, 4], [5, 2]]
    filters = w.float().t().contiguous().to(DEV)
    at = [0] * 4
    for step in SCHEDULE:
        x = torch.cat([u[i][at[i]:at[i] + n] for i, n in enumerate(step)])
        pad = torch.zeros(len(x), c + (-c) % 8 + 8, dtype=dtype, device=DEV)
        pad[:, :c] = x.to(DEV)
        slots = [pages[i][p // 64] * 64 + p % 64 for i, n in enumerate(step)
                 for p in range(at[i], at[i] + n)]
        if all(n == 1 for n in step):
            conv = (None, None, None, i32(*[a + 1 for a in at]), None,
                    i32(4, 3, 2, 1))
        else:
            conv = _steps(step, at)
        q = D.conv_qkv(pad[:, :c], filters, tails, rope.cos, rope.sin, rot,
                       i32(*slots), kc, vc, H, *conv)
        close(q, torch.cat([want[i][0][at[i]:at[i] + n]
                            for i, n in enumerate(step)]), dtype)
        at = [a + n for a, n in zip(at, step)]
    for i, n in enumerate(total):
        p = torch.tensor([pages[i][t // 64] for t in range(n)])
        o = torch.arange(n) % 64
        close(kc.cpu()[p, :, o].reshape(n, -1), want[i][1].reshape(n, -1),
              dtype)
        close(vc.cpu()[p, :, o].reshape(n, -1), want[i][2].reshape(n, -1),
              dtype)
    # a row that is not in use leaves everything alone
    before = tails.clone(), kc.clone(), vc.clone()
    D.conv_qkv(pad[:4, :c], filters, tails, rope.cos, rope.sin, rot,
               i32(-1, -1, -1, -1), kc, vc, H, None, None, None,
               i32(0, 0, 0, 0), None, i32(-1, -1, -1, -1))
    for a, b in zip(before, (tails, kc, vc)):
        assert torch.equal(a.nan_to_num(9.0), b.nan_to_num(9.0))


@BOTH
@pytest.mark.parametrize("taps", [1, 2, 4, 6])
@pytest.mark.parametrize("c", [10, 36, 264])
def test_conv_silu(c, taps, dtype):
    g = gen(c)
    total = [sum(s[i] for s in SCHEDULE) for i in range(4)]
    u = [rnd(g, t, c, dtype=dtype) for t in total]
    w, b = rnd(g, c, taps, dtype=BF), rnd(g, c)
    want = [O.silu(O.short_conv(x.double(), w.double(), b.double()))
            for x in u]
    tails = torch.full((6, taps - 1, c), float("nan"), dtype=dtype,
                       device=DEV)
    at = [0] * 4
    for step in SCHEDULE:
        x = torch.cat([u[i][at[i]:at[i] + n] for i, n in enumerate(step)])
        conv = _steps(step, at) if max(step) > 1 else \
            (None, None, None, i32(*[a + 1 for a in at]), None,
             i32(4, 3, 2, 1))
        got = D.conv_silu(x.to(DEV), w.float().t().contiguous().to(DEV),
                          b.to(DEV), tails, *conv)
        close(got, torch.cat([want[i][at[i]:at[i] + n]
                              for i, n in enumerate(step)]), dtype)
        at = [a + n for a, n in zip(at, step)]


# ---- attention --------------------------------------------------------------

@BOTH
@pytest.mark.parametrize("H,G,Dm,E", [
    (3, 3, 20, 18), (6, 2, 40, 72), (17, 1, 32, 32), (40, 2, 64, 48),
    (8, 2, 128, 128), (4, 1, 256, 136), (2, 1, 72, 256), (4, 4, 24, 16)])
def test_grouped_attention(H, G, Dm, E, dtype):
    """Rows and portions over a scattered page table whose other pages and
    unused places hold garbage; some rows single out one key at a page's edge,
    the first, or one far back."""
    g = gen(Dm + E)
    T, scale = 300, 0.8 * Dm ** -0.5
    q, k, v = (rnd(g, T, n, d, dtype=dtype)
               for n, d in ((H, Dm), (G, Dm), (G, E)))
    sink = rnd(g, H) + 1.0
    gate = rnd(g, T, H * E, dtype=dtype)
    for row, key in ((299, 0), (298, 63), (297, 64), (296, 127), (295, 128),
                     (130, 129), (200, 5), (64, 63), (65, 64)):
        for h in range(H):
            q[row, h] = (k[key, h // (H // G)].float() * 3).to(dtype)
    pages = [7, 2, 9, 4, 1]
    kc = torch.full((11, G, 64, Dm), 50.0, dtype=dtype)
    vc = torch.full((11, G, 64, E), float("nan"), dtype=dtype)
    for t in range(T):
        kc[pages[t // 64], :, t % 64] = k[t]
        vc[pages[t // 64], :, t % 64] = v[t]
    kc, vc = kc.to(DEV), vc.to(DEV)
    bt = torch.tensor([[0] * 5, pages], dtype=torch.int32, device=DEV)
    plain = O.sink_attention(q.double(), k.double(), v.double(), scale,
                             sink.double()).reshape(T, -1)
    want = plain * O.sigmoid(gate.double()) * 0.7
    qf = q.reshape(T, -1)
    some = [0, 1, 62, 63, 64, 65, 127, 128, 130, 190, 191, 200, 250, 295, 296,
            297, 298, 299]
    idx = torch.tensor(some)
    for row_item, table in ((i32(*[1] * len(some)), bt),
                            (None, bt[1:].repeat(len(some), 1))):
        out = torch.zeros(len(some), H * E + 8, dtype=dtype, device=DEV)
        D.gqa_rows(qf[idx].to(DEV), kc, vc, table, row_item,
                   (idx + 1).int().to(DEV), sink.to(DEV), gate[idx].to(DEV),
                   out[:, :H * E], H, scale, 0.7)
        close(out[:, :H * E], want[idx], dtype)
        assert not out[:, H * E:].any()
    # without sink and gate
    bare = O.sink_attention(q.double(), k.double(), v.double(), scale,
                            torch.full((H,), -1e30).double()).reshape(T, -1)
    out = torch.zeros(len(some), H * E, dtype=dtype, device=DEV)
    D.gqa_rows(qf[idx].to(DEV), kc, vc, bt, i32(*[1] * len(some)),
               (idx + 1).int().to(DEV), None, None, out, H, scale)
    close(out, bare[idx], dtype)
    # rows not in use come out as zero, without reading anything
    off = torch.ones(2, H * E, dtype=dtype, device=DEV)
    D.gqa_rows(qf[:2].to(DEV), kc, vc, bt, None, i32(0, 0), sink.to(DEV),
               None, off, H, scale)
    assert not off.any()
    if dtype != BF or not D.gqa_mfma_ok(Dm, E):
        return
    block = D.gqa_portion_rows(Dm, E)
    for start, n in ((0, 300), (63, 2), (64, 65), (130, 170), (200, 64),
                     (1, 128)):
        for s, gt, ref in ((sink.to(DEV), gate, want), (None, None, bare)):
            out = torch.empty(n, H * E, dtype=dtype, device=DEV)
            t0 = list(range(0, n, block))[::-1]
            D.gqa_portions(
                qf[start:start + n].to(DEV), kc, vc, bt[1:], s,
                None if gt is None else gt[start:start + n].to(DEV),
                i32(*[0] * len(t0)), i32(*t0), i32(0), i32(start), i32(n),
                out, H, scale, 0.7 if gt is not None else 1.0)
            close(out, ref[start:start + n], dtype)


def test_portions_of_several_sequences():
    """One launch over portions of two sequences, rows behind each other."""
    g = gen(9)
    H, G, Dm, E, scale = 4, 2, 32, 48, 0.3
    lens, starts = [70, 150], [40, 0]
    bt = torch.tensor([[3, 0, 0], [5, 1, 4]], dtype=torch.int32)
    bt[0, 1] = 2
    kc = torch.zeros(6, G, 64, Dm, dtype=BF)
    vc = torch.zeros(6, G, 64, E, dtype=BF)
    q, want = [], []
    for i, (n, st) in enumerate(zip(lens, starts)):
        T = st + n
        qq, k, v = (rnd(g, T, m, d, dtype=BF)
                    for m, d in ((H, Dm), (G, Dm), (G, E)))
        for t in range(T):
            kc[bt[i, t // 64], :, t % 64] = k[t]
            vc[bt[i, t // 64], :, t % 64] = v[t]
        want.append(O.sink_attention(qq.double(), k.double(), v.double(),
                                     scale, torch.zeros(H).double())
                    [st:].reshape(n, -1))
        q.append(qq[st:].reshape(n, -1))
    block = D.gqa_portion_rows(Dm, E)
    item = [i for i, n in enumerate(lens) for _ in range(0, n, block)]
    t0 = [t for n in lens for t in range(0, n, block)]
    out = torch.empty(sum(lens), H * E, dtype=BF, device=DEV)
    D.gqa_portions(torch.cat(q).to(DEV), kc.to(DEV), vc.to(DEV), bt.to(DEV),
                   torch.zeros(H, device=DEV), None, i32(*item), i32(*t0),
                   i32(0, lens[0]), i32(*starts), i32(*lens), out, H, scale)
    close(out, torch.cat(want), BF)


# ---- state space ------------------------------------------------------------

SSD_SHAPES = [(3, 7, 13, 1), (4, 16, 8, 2), (2, 40, 48, 1), (6, 24, 32, 3),
              (4, 64, 128, 2), (2, 136, 96, 2), (1, 256, 256, 1),
              (5, 8, 64, 5)]


@BOTH
@pytest.mark.parametrize("H,P,N,G", SSD_SHAPES)
def test_ssd_kernels(H, P, N, G, dtype):
    """Portions (token loop and chunks) and single tokens, carrying the state
    from one to the next, with heads that forget at once and ones that
    hardly do."""
    g = gen(H * P)
    lens = [150, 64, 1, 2, 65, 3, 1]
    T, inner = sum(lens), H * P
    cx, zo = inner + 2 * G * N, 8
    dto = zo + inner + (-inner) % 8
    xbc = rnd(g, T, cx, dtype=dtype)
    u = rnd(g, T, dto + H + (-(dto + H)) % 8, dtype=dtype)
    A = torch.tensor([0.02, 8.0, 1.0, 300.0, 0.0, 0.3])[:H].contiguous()
    bias = torch.tensor([-1.0, 0.5, -3.0, 1.0, -2.0, 4.0])[:H].contiguous()
    skip = rnd(g, H)
    dt = O.softplus(u[:, dto:dto + H].double() + bias.double())
    z = u[:, zo:zo + inner].double()
    x = xbc[:, :inner].double().reshape(T, H, P)
    B, Cm = (xbc[:, inner + i * G * N:inner + (i + 1) * G * N].double()
             .reshape(T, G, N) for i in range(2))
    const = (A.to(DEV), bias.to(DEV), skip.to(DEV))
    for chunked in ([False, True] if dtype == BF else [False]):
        if chunked and not D.ssd_chunked_ok(H, N, P, G):
            continue
        state = torch.full((3, H, N, P), float("nan"), device=DEV)
        S, at = None, 0
        for n in lens:
            part = u[at:at + n].to(DEV), xbc[at:at + n].to(DEV)
            if n == 1:
                out = D.ssd_decode(part[0], zo, dto, part[1], *const, state,
                                   G, i32(2), i32(at + 1))
            else:
                out = torch.empty(n, inner, dtype=dtype, device=DEV)
                items = i32(2), i32(0), i32(at), i32(n)
                if chunked:
                    nch = -(-n // 64)
                    D.ssd_chunked(part[0], zo, dto, part[1], *const, state,
                                  G, *items, i32(0), i32(*[0] * nch),
                                  i32(*range(0, n, 64)), out)
                else:
                    D.ssd_seq(part[0], zo, dto, part[1], *const, state, G,
                              *items, out)
            r = slice(at, at + n)
            y, S = O.ssd_recurrence(x[r], B[r], Cm[r], dt[r], A.double(),
                                    skip.double(), S)
            close(out, y.reshape(n, inner) * O.silu(z[r]), dtype)
            # the state itself is f32-accurate on every path
            got = state[2].double().cpu()
            assert float((got - S).abs().max() /
                         S.pow(2).mean().sqrt()) < 3e-4
            at += n
    # rows not in use come out as zero and touch no state
    before = state.clone()
    out = D.ssd_decode(u[:2].to(DEV), zo, dto, xbc[:2].to(DEV), *const, state,
                       G, i32(-1, -1), i32(0, 0))
    assert not out.any()
    assert torch.equal(before.nan_to_num(9.0), state.nan_to_num(9.0))


# ---- the model through the framework ----------------------------------------

@pytest.fixture(scope="module")
def cases():
    return {(n, t): C.Case(n, DEV, t) for n in C.CONFIGS for t in (F32, BF)}


NAMES = pytest.mark.parametrize("name", list(C.CONFIGS))


@BOTH
@NAMES
def test_residual_after_every_layer(cases, name, dtype):
    case = cases[name, dtype]
    toks = case.tokens(90)
    kv = case.model.new_kv_cache(2, 1)
    kv.allocate(0, 90)
    trail = []
    case.model.forward_prefill_batch(
        [(torch.tensor(toks, device=DEV), 0, 0)], kv, trail=trail)
    want = O.forward(case.raw, case.weights, toks)[1]
    assert len(trail) == len(want)
    for a, b in zip(trail, want):
        err = (a.double().cpu() - b).pow(2).mean().sqrt() / \
            b.pow(2).mean().sqrt()
        assert float(err) < (2e-5 if dtype == F32 else 2e-2)


@BOTH
@NAMES
@pytest.mark.parametrize("cuts", list(C.CUTS))
def test_cuts(cases, name, cuts, dtype):
    C.scenario_cuts(cases[name, dtype], 150, cuts)


@BOTH
@NAMES
def test_mixed_batches(cases, name, dtype):
    for seed in range(2):
        C.scenario_mixed(cases[name, dtype], seed)


@BOTH
@NAMES
def test_slot_and_page_reuse(cases, name, dtype):
    C.scenario_reuse(cases[name, dtype])


@BOTH
@pytest.mark.parametrize("spot,n", [(0, 200), (63, 150), (64, 200)])
@pytest.mark.parametrize("cuts", [
    lambda n: [n], lambda n: [n - 12] + [1] * 12,
    lambda n: C.portions(n, [2, 37])], ids=["prompt", "decoded", "portions"])
def test_far_keys(spot, n, cuts, dtype):
    C.scenario_far_key(spot, n, DEV, dtype, cuts)


@BOTH
def test_long_prompt_and_long_decoding(cases, dtype):
    case = cases["ones", dtype]
    C.scenario_cuts(case, 1000, "whole")
    C.scenario_cuts(case, 700, "decoded tail")


@BOTH
@pytest.mark.parametrize("chunk", [None, 24])
@pytest.mark.parametrize("graph", [True, False])
@pytest.mark.parametrize("name", ["odd", "tiles"])
def test_generation(cases, name, chunk, graph, dtype):
    C.scenario_generate(cases[name, dtype], use_graph=graph,
                        chunk_tokens=chunk)


@BOTH
def test_graph_replays_match_eager_steps(cases, dtype):
    """Captured decode runs, several in a row with eager work between them,
    against eager decoding of the same prompts."""
    case = cases["tiles", dtype]
    prompts = [case.tokens(n, seed=n) for n in (70, 3, 129)]
    eng = case.engine(1024)
    ref = case.engine(1024)
    ref.use_graph = False
    for again in range(3):
        a = eng.generate_batch(prompts, [20, 20, 20])
        assert eng.use_graph and not eng._graph_failed
        b = ref.generate_batch(prompts, [20, 20, 20])
        if dtype == F32:
            assert a == b
        for p, o in zip(prompts, a):
            C.greedy_check(case, p, o)
        torch.zeros(64, 1024, device=DEV).normal_().sum().item()


@BOTH
def test_conversations_reuse_the_snapshot(cases, dtype):
    C.scenario_conversation(cases["tiles", dtype])


def test_preset_on_engine():
    from quickstart_streaming_agents_amd.models import build_model
    from quickstart_streaming_agents_amd.models.serve import Engine, EngineLLM
    llm = EngineLLM(Engine(build_model("tiny-lunulix", device=DEV),
                           max_batch=4, max_seq_len=512))
    out = llm(["price of boots?", "hello"], [8, 8], ["a", "b"])
    assert len(out) == 2
    llm.release_all()
    assert llm.engine.kv.free_slots == llm.engine.kv.n_slots
