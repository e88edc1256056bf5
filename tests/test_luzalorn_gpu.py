"""Luzalorn on the GPU: every kernel against plain f32/f64 references of the
same mechanism, then the model through the framework's step function, cache,
scheduler and graph against the oracle, in f32 and bf16."""

import luzalorn_cases as C
import luzalorn_oracle as O
import pytest
import torch

from quickstart_streaming_agents_amd.ops import dispatch as D

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
F32, BF = torch.float32, torch.bfloat16


def gen(seed):
    return torch.Generator().manual_seed(seed)


def rnd(g, *shape, dtype=F32, scale=1.0):
    return (torch.randn(*shape, generator=g) * scale).to(dtype)


def close(got, want, dtype):
    """Largest rms error of a row, relative to the rms of everything."""
    got, want = got.double().cpu(), want.double()
    rms = want.pow(2).mean().sqrt().clamp(min=1e-6)
    err = (got - want).pow(2).mean(-1).sqrt().max() / rms
    assert float(err) <= (2e-5 if dtype == F32 else 3e-2), float(err)


# ---- kernels ----------------------------------------------------------------

@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("W", [33, 100, 256, 4096, 8448])
def test_residual_norm(W, dtype):
    g = gen(W)
    T, V = 7, 11
    res, y = rnd(g, T, W), rnd(g, T, W, dtype=dtype)
    table, ids = rnd(g, V, W, dtype=dtype), torch.tensor([0, 10, 3, 3, 1, 9, 2])
    vec, w, b = (rnd(g, W, dtype=dtype) for _ in range(3))
    for init, layer, full in ((True, True, True), (False, True, False),
                              (False, False, True)):
        r = res.to(DEV)
        out = D.residual_norm(
            r, y.to(DEV), w.to(DEV), b.to(DEV) if layer else None, 1e-4,
            table=table.to(DEV) if full else None,
            ids=ids.to(DEV) if full else None,
            vec=vec.to(DEV) if full else None, init=init, layer=layer)
        x = (0 if init else res.double()) + y.double()
        if full:
            x = x + table.double()[ids] + vec.double()
        close(r, x, F32)
        want = O.layer_norm(x, w.double(), b.double(), 1e-4) if layer \
            else O.rms(x, 1e-4, w.double())
        close(out, want, dtype)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("cols", [5, 90, 264])
def test_glu(cols, dtype):
    x = rnd(gen(1), 19, 2 * cols, dtype=dtype, scale=3.0)
    d = x.to(DEV)
    got = D.glu(d[:, :cols], d[:, cols:])
    close(got, O.silu(x[:, :cols].double()) * x[:, cols:].double(), dtype)


def test_argmax_rows():
    for dtype in (F32, BF):
        x = rnd(gen(2), 9, 5000, dtype=dtype)
        x[3, 77] = x[3, 4001] = 90.0
        got = D.argmax_rows(x.to(DEV)).cpu()
        assert int(got[3]) == 77
        assert torch.equal(x.float().gather(1, got[:, None])[:, 0],
                           x.float().max(-1).values)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("M,H,N,K", [(1, 3, 36, 20), (5, 2, 72, 96),
                                     (70, 4, 512, 128), (33, 17, 40, 24)])
def test_head_matmul(M, H, N, K, dtype):
    g = gen(M)
    x = rnd(g, M, H * K + 8, dtype=dtype)
    w = rnd(g, H, N, K, dtype=dtype, scale=K ** -0.5)
    gate = rnd(g, M, H * N, dtype=dtype)
    want = torch.stack([x[:, h * K:(h + 1) * K].double() @ w[h].double().T
                        for h in range(H)], 1).reshape(M, H * N)
    xs = x.to(DEV)[:, :H * K]
    close(D.head_matmul(xs, w.to(DEV)), want, dtype)
    close(D.head_matmul(xs, w.to(DEV), gate.to(DEV)),
          want * O.sigmoid(gate.double()), dtype)


def _rotated(x, pos0, m):
    T, H, Dm, E = x.shape[0], m["heads"], m["dim"], m["vdim"]
    pos = pos0 + torch.arange(T).double()
    q = x[:, :H * Dm].double().reshape(T, H, Dm)
    k = x[:, H * Dm:2 * H * Dm].double().reshape(T, H, Dm)
    v = x[:, 2 * H * Dm:2 * H * Dm + H * E].double().reshape(T, H, E)
    gate = x[:, 2 * H * Dm + H * E:].double()
    rot = m["rot"]
    return (O.rotate(q, pos, rot["dims"], rot["base"]),
            O.rotate(k, pos, rot["dims"], rot["base"]) * Dm ** -0.5, v, gate)


RET_SHAPES = [(3, 20, 28, 12), (2, 32, 64, 32), (2, 48, 80, 32),
              (3, 64, 24, 64), (1, 128, 256, 128), (1, 256, 320, 128),
              (2, 96, 512, 64)]


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("H,Dm,E,rot", RET_SHAPES)
def test_retention_kernels(H, Dm, E, rot, dtype):
    """Portions (token loop and chunks) and single tokens, carrying the
    state from one to the next, with a decay of one and a fast one."""
    from quickstart_streaming_agents_amd.models.layers import RopeTable
    decay = [1.0, 0.3, 0.996][:H]
    m = C.ret(H, Dm, E, rot, decay)["mixer"]
    table = RopeTable(rot, 10_000.0, DEV)
    table.ensure(600)
    dec = torch.tensor(decay).to(DEV)
    l2 = torch.log2(torch.tensor(decay, dtype=torch.float64)).float().to(DEV)
    g = gen(Dm)
    lens, width = [150, 64, 1, 2, 65, 3], 2 * H * (Dm + E)
    pad = width + (-width) % 8
    x = rnd(g, sum(lens), pad, dtype=dtype)[:, :width]
    # one sequence in six steps; portions by both prefill kernels
    for chunked in ([False, True] if dtype == BF else [False]):
        if chunked and not D.retention_chunked_ok(H, Dm, E):
            continue
        state = torch.full((3, H, Dm, E), float("nan"), device=DEV)
        S, at = None, 0
        for n in lens:
            part = torch.zeros(n, pad, dtype=dtype, device=DEV)
            part[:, :width] = x[at:at + n].to(DEV)
            xs = part[:, :width]
            i32 = lambda *v: torch.tensor(v, dtype=torch.int32, device=DEV)
            args = (xs, table.cos, table.sin)
            if n == 1:
                out = D.retention_decode(*args, dec, state, i32(2),
                                         i32(at + 1), rot, Dm ** -0.5, 1e-5)
            else:
                out = torch.empty(n, H * E, dtype=dtype, device=DEV)
                if chunked:
                    nch = -(-n // 64)
                    D.retention_chunked(
                        *args, l2, state, i32(2), i32(0), i32(at), i32(n),
                        i32(*range(at, at + n)), i32(0), i32(*[0] * nch),
                        i32(*range(0, n, 64)), out, rot, Dm ** -0.5, 1e-5)
                else:
                    D.retention_seq(*args, dec, state, i32(2), i32(0),
                                    i32(at), i32(n), out, rot, Dm ** -0.5,
                                    1e-5)
            q, k, v, gate = _rotated(x[at:at + n], at, m)
            o, S = O.retention_recurrence(q, k, v, decay, S)
            want = O.rms(o, 1e-5).reshape(n, H * E) * O.silu(gate)
            close(out, want, dtype)
            # the state itself is f32-accurate on every path
            got = state[2].double().cpu()
            assert float((got - S).abs().max() /
                         S.pow(2).mean().sqrt()) < 3e-4
            at += n


def _attention_reference(q, c, uk, uv, scale, window, sink, gate, start):
    """rows of q [n, H, D] at positions start.. over latents c [T, R]"""
    n, H, Dm = q.shape
    T = c.shape[0]
    k = (c @ uk.reshape(-1, c.shape[1]).T).view(T, H, Dm)
    v = (c @ uv.reshape(-1, c.shape[1]).T).view(T, H, -1)
    qq = torch.zeros(T, H, Dm, dtype=torch.float64)
    qq[start:start + n] = q
    o = O.window_softmax_attention(qq, k, v, scale, window or None, sink)
    return o[start:start + n].reshape(n, -1) * O.sigmoid(gate)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("H,Dm,E,R,window", [
    (3, 20, 18, 36, 70), (5, 40, 72, 96, 0), (16, 32, 32, 64, 64),
    (17, 128, 136, 512, 190), (2, 16, 256, 200, 1), (4, 256, 16, 24, 65)])
def test_latent_attention_kernels(H, Dm, E, R, window, dtype):
    """Absorbed rows and expanded portions over a scattered page table,
    rows at page and window edges, one key far above the others."""
    g = gen(R)
    T, scale = 300, 0.8 * Dm ** -0.5
    c = rnd(g, T, R, dtype=dtype)
    uk = rnd(g, H, Dm, R, dtype=dtype, scale=R ** -0.5)
    uv = rnd(g, H, E, R, dtype=dtype, scale=R ** -0.5)
    sink = rnd(g, H, dtype=dtype)
    q = rnd(g, T, H * Dm, dtype=dtype)
    q[250:] = 6 * q[250:]                  # these rows look at few keys
    gate = rnd(g, T, H * E, dtype=dtype)
    pages = [7, 2, 9, 4, 1]
    cache = torch.full((11, 64, R), 50.0, dtype=dtype)
    for i, p in enumerate(pages):
        rows = c[i * 64:(i + 1) * 64]
        cache[p, :len(rows)] = rows
    cache = cache.to(DEV)
    bt = torch.tensor([[0] * 5, pages], dtype=torch.int32, device=DEV)
    want = _attention_reference(
        q.double().view(T, H, Dm), c.double(), uk.double(), uv.double(),
        scale, window, sink.double(), gate.double(), 0)
    some = [0, 1, 62, 63, 64, 65, 127, 128, 189, 190, 191, 249, 250, 299]
    idx = torch.tensor(some)
    qa = D.head_matmul(q[idx].to(DEV), uk.transpose(1, 2).contiguous().to(DEV))
    lat = D.latent_rows(
        qa, cache, bt, torch.ones(len(some), dtype=torch.int32, device=DEV),
        (idx + 1).int().to(DEV), sink.to(DEV), window, scale)
    got = D.head_matmul(lat, uv.to(DEV), gate[idx].to(DEV))
    close(got, want[idx], dtype)
    # rows not in use come out as zero, without reading anything
    off = D.latent_rows(qa[:2].contiguous(), cache, bt, None,
                        torch.zeros(2, dtype=torch.int32, device=DEV),
                        sink.to(DEV), window, scale)
    assert not off.any()
    if dtype != BF or not D.window_attn_ok(H, Dm, E) or R % 8:
        return
    w = torch.cat([uk.view(-1, R), uv.view(-1, R)]).to(DEV)
    i32 = lambda *v: torch.tensor(v, dtype=torch.int32, device=DEV)
    for start, n in ((0, 300), (63, 2), (64, 65), (130, 170), (200, 64)):
        first = max(0, start - window + 1) if window else 0
        kv = c[first:start + n].to(DEV) @ w.T
        out = torch.empty(n, H * E, dtype=dtype, device=DEV)
        nb = -(-n // 64)
        D.window_attn_prefill(
            q[start:start + n].to(DEV), kv, gate[start:start + n].to(DEV),
            sink.to(DEV), i32(*[0] * nb), i32(*range(0, n, 64)), i32(0),
            i32(start), i32(n), i32(0), i32(first), out, Dm, E, window, scale)
        close(out, want[start:start + n], dtype)


def test_latent_norm_store_and_slots():
    for dtype in (F32, BF):
        g = gen(5)
        x = rnd(g, 6, 100, dtype=dtype)
        wq, wk = rnd(g, 52, dtype=dtype), rnd(g, 36, dtype=dtype)
        cache = torch.zeros(4, 64, 36, dtype=dtype, device=DEV)
        bt = torch.tensor([[3, 0], [1, 2], [0, 0], [2, 1], [1, 1], [0, 3]],
                          dtype=torch.int32, device=DEV)
        lens = torch.tensor([1, 65, 0, 64, 3, 128], dtype=torch.int32,
                            device=DEV)
        slots = D.decode_slots(bt, lens)
        assert slots.tolist() == [192, 128, -1, 191, 66, 255]
        cq = D.latent_norm_store(x.to(DEV), wq.to(DEV), wk.to(DEV), cache,
                                 slots, 1e-5)
        close(cq, O.rms(x[:, :52].double(), 1e-5, wq.double()), dtype)
        want = O.rms(x[:, 52:88].double(), 1e-5, wk.double())
        flat = cache.view(-1, 36)
        for r, s in enumerate(slots.tolist()):
            if s >= 0:
                close(flat[s], want[r], dtype)
        assert int((flat != 0).any(-1).sum()) == 5


# ---- the model through the framework ----------------------------------------

@pytest.fixture(scope="module")
def cases():
    return {(n, t): C.Case(n, DEV, t) for n in C.CONFIGS for t in (F32, BF)}


DTYPES = pytest.mark.parametrize("dtype", [F32, BF], ids=["f32", "bf16"])
NAMES = pytest.mark.parametrize("name", list(C.CONFIGS))


@DTYPES
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
    for a, b in zip(trail, want):
        err = (a.double().cpu() - b).pow(2).mean().sqrt() / \
            b.pow(2).mean().sqrt()
        assert float(err) < (2e-5 if dtype == F32 else 2e-2)


@DTYPES
@NAMES
@pytest.mark.parametrize("cuts", list(C.CUTS))
def test_cuts(cases, name, cuts, dtype):
    C.scenario_cuts(cases[name, dtype], 150, cuts)


@DTYPES
@NAMES
def test_mixed_batches(cases, name, dtype):
    for seed in range(2):
        C.scenario_mixed(cases[name, dtype], seed)


@DTYPES
@NAMES
def test_slot_and_page_reuse(cases, name, dtype):
    C.scenario_reuse(cases[name, dtype])


@DTYPES
@pytest.mark.parametrize("window", [1, 63, 64, 65])
@pytest.mark.parametrize("cuts", [
    lambda n: [n], lambda n: [n - 60] + [1] * 60,
    lambda n: C.portions(n, [2, 37])], ids=["prompt", "decoded", "portions"])
def test_window_edges(window, cuts, dtype):
    C.scenario_window_edge(window, DEV, dtype, cuts)


@DTYPES
def test_long_prompt_and_long_decoding(cases, dtype):
    case = cases["ones", dtype]
    C.scenario_cuts(case, 1000, "whole")
    C.scenario_cuts(case, 700, "decoded tail")


@DTYPES
@pytest.mark.parametrize("chunk", [None, 24])
@pytest.mark.parametrize("graph", [True, False])
@pytest.mark.parametrize("name", ["odd", "tiles"])
def test_generation(cases, name, chunk, graph, dtype):
    C.scenario_generate(cases[name, dtype], use_graph=graph,
                        chunk_tokens=chunk)


@DTYPES
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


@DTYPES
def test_conversations_reuse_the_snapshot(cases, dtype):
    C.scenario_conversation(cases["tiles", dtype])


def test_llama_chunked_prefill_on_gpu():
    from quickstart_streaming_agents_amd.models import build_model
    from quickstart_streaming_agents_amd.models.serve import Engine
    model = build_model("tiny", device=DEV, seed=3)
    prompts = [[1, 5, 9, 13] * 30, [2, 4, 6], [7] * 65]
    outs = Engine(model, max_batch=2, max_seq_len=256,
                  chunk_tokens=40).generate_batch(prompts, [6, 9, 5])
    assert [len(o) for o in outs] == [6, 9, 5]


def test_preset_on_engine():
    from quickstart_streaming_agents_amd.models import build_model
    from quickstart_streaming_agents_amd.models.serve import Engine, EngineLLM
    llm = EngineLLM(Engine(build_model("tiny-luzalorn", device=DEV),
                           max_batch=4, max_seq_len=512))
    out = llm(["price of boots?", "hello"], [8, 8], ["a", "b"])
    assert len(out) == 2
    llm.release_all()
    assert llm.engine.kv.free_slots == llm.engine.kv.n_slots
