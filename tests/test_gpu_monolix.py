"""Monolix through the engine on the GPU against the CPU oracle (float64, one sequence at a time, no cache): single
mechanisms, kernels on crafted inputs (a far key among hundreds, a tempting key one position ahead, choice scores of either
sign), whole prompts with the stream after every layer, decoding through the cache, portions down to two tokens, unequal
batches, reused rows and slots, graph replay, other sizes, and generation through the engine's scheduler.

Sharp comparisons run the engine in fp32 (the oracle's weights are bf16-representable, so both see the same numbers); a
bf16 pass checks the serving precision against a looser bar."""
import pytest
import torch

from oracle import monolix as mo
from tests import monolix_util as U
from tests.test_gpu_toredra import engine, entry, portions, run_portions, run_whole, seq_params

pytestmark = pytest.mark.gpu
F32_BAR = 2e-4


# ------------------------------------------------------------------------------------------------ mechanisms alone
LAYERS = [
    (U.attention(4, 2, 16, dims=8), None),
    (U.attention(3, 3, 24, scale=0.5), None),                              # kv heads = heads, rotation over the whole head
    (U.attention(5, 1, 72, dims=0), None),                                 # no rotation, one kv head
    (U.attention(2, 1, 200, dims=72, scale=0.05), None),                   # heads above 128
    (U.attention(1, 1, 10, dims=6, base=3.0), None),                       # a width no vector load divides
    (U.attention(2, 2, 16), U.moe(6, 2, 40)), (U.attention(2, 1, 16), U.moe(4, 1, 24, identity=4, shared=40)),
    (U.attention(2, 2, 16), U.moe(5, 3, 16, identity=7, count=4, keep=2)), (U.attention(1, 1, 16), U.moe(2, 3, 16, 1, shared=8)),
    (U.attention(2, 2, 16), U.moe(9, 3, 30, identity=3, count=4, keep=1, shared=33)),
]


@pytest.mark.parametrize("layer", range(len(LAYERS)))
@pytest.mark.parametrize("W", [80, 77])
def test_single_layer_models_match_oracle(tmp_path, layer, W):
    cfg = U.config([LAYERS[layer]], width=W)
    folder, w = U.make_model(tmp_path, cfg, seed=5)
    toks = U.tokens(70, cfg["vocab"], 6)
    eng = engine(folder)
    eng.runner.model.capture_layers = []
    got = run_whole(eng, toks)
    lay = []
    want = mo.forward(toks, w, cfg, lay)
    assert U.rel(eng.runner.model.capture_layers[0], lay[0]) < F32_BAR
    assert U.rel(got, want) < F32_BAR


# ------------------------------------------------------------------------------------------------ row kernels
@pytest.mark.parametrize("W", [200, 77, 1544, 3072, 4100])
@pytest.mark.parametrize("alpha", [1.0, 2.5])
def test_post_norm_kernel_in_every_form(W, alpha):
    """the sum with a result, with a mixture (experts, identity experts, both), with and without a dense branch and its gate;
    rows of the mixture that belong to no expert hold NaN and must not be read"""
    from scratchpad_amd import _native
    g = torch.Generator().manual_seed(0)
    T, top, E, eps = 19, 3, 5, 1e-5
    rn = lambda *s: torch.randn(*s, generator=g)
    x, a, z = rn(T, W) * torch.linspace(0.1, 9.0, W), rn(T, 2 * W) * 3, rn(T * top, W) * 2
    weight, scale, gate, wts = 1 + 0.3 * rn(W), 1 + 0.5 * rn(W), torch.rand(T, generator=g), torch.rand(T, top, generator=g)
    ids = torch.stack([torch.randperm(9, generator=g)[:top] for _ in range(T)]).to(torch.int32)
    ids[0], ids[1] = torch.tensor([0, 1, 4]), torch.tensor([5, 8, 6])                # all experts, all identity
    place = torch.randperm(T * top, generator=g).to(torch.int32)
    z[place.long()[(ids >= E).flatten()]] = float("nan")
    c = lambda t: None if t is None else t.cuda()
    for dtype, bar in ((torch.float32, 2e-6), (torch.bfloat16, 1e-2)):
        r = lambda t: t.to(dtype).double()
        for form in ("plain", "unscaled", "mix", "mix+dense", "mix+gate"):
            y = r(a[:, W:]) if form in ("plain", "unscaled", "mix+dense") else (gate.double()[:, None] * r(a[:, W:]) if form == "mix+gate" else 0)
            if form.startswith("mix"):
                rows = torch.where((ids >= E)[..., None], x.double()[:, None], r(z)[place.long().view(T, top)])
                y = y + (wts.double()[..., None] * rows).sum(1)
            s = None if form == "unscaled" else scale
            want = mo.rms(alpha * x.double() + (1 if s is None else s.double()) * y, eps) * weight.double()
            mix = dict(z=z.to(dtype).cuda(), ids=c(ids), place=c(place), weights=c(wts), experts=E) if form.startswith("mix") else {}
            for want_lo in (True, False):
                xs = x.clone().cuda()
                out = _native.post_norm(xs, None if form == "mix" else a.to(dtype).cuda()[:, W:], c(weight), eps, alpha, dtype,
                                        scale=c(s), gate=c(gate) if form == "mix+gate" else None, want_lo=want_lo, **mix)
                assert U.rel(xs, want) < 3e-6, (dtype, form)
                if want_lo:
                    assert out.dtype == dtype and torch.equal(out, xs.to(dtype)), (dtype, form)
                else:
                    assert out is None


@pytest.mark.parametrize("E,top,count,keep", [(14, 3, 2, 1), (12, 4, 6, 2), (5, 5, 1, 1), (70, 1, 1, 1), (130, 6, 65, 4),
                                              (9, 3, 9, 3), (8, 2, 4, 4)])
def test_router_choice_in_groups_with_corrections_of_either_sign(E, top, count, keep):
    from scratchpad_amd import _native
    g = torch.Generator().manual_seed(1)
    x, W = torch.randn(90, 24, generator=g), torch.randn(E + 1, 24, generator=g) * 0.6
    for shift in (0.0, -2.0):                                     # -2: every choice score is negative
        corr = 0.2 * torch.randn(E, generator=g) + shift
        w = {"r.router": W[:E].double(), "r.correction": corr.double()}
        wi, ww = mo.route(x.double(), w, "r", U.moe(E, top, 8, 0, count, keep)["router"])
        for n in (90, 7):                                         # the library's fp32 product, the own kernel
            ids, wt, gate = _native.moe_route_softmax(x[:n].cuda(), W.cuda(), top, 1.0, correction=corr.cuda(), groups=count,
                                                      keep=keep, gate_row=True)
            assert torch.equal(ids.cpu().long(), wi[:n]) and U.rel(wt, ww[:n]) < 1e-5
            assert U.rel(gate, torch.sigmoid(x[:n].double() @ W[E].double())) < 1e-5


@pytest.mark.parametrize("dtype,bar", [(torch.float32, 2e-6), (torch.bfloat16, 1e-2)], ids=["fp32", "bf16"])
@pytest.mark.parametrize("W,ff,T", [(64, 96, 50), (72, 40, 7), (128, 64, 1)])
def test_expert_rows_leave_out_the_identity_pairs(dtype, bar, W, ff, T):
    from scratchpad_amd.moe import ReluSquareExperts
    g = torch.Generator().manual_seed(2)
    E, outputs, top = 4, 7, 3
    ex = ReluSquareExperts(W, E, ff, dtype=dtype).cuda()
    ex.up.data.copy_(torch.randn(E, ff, W, generator=g) * W ** -0.5)
    ex.down.data.copy_(torch.randn(E, W, ff, generator=g) * ff ** -0.5)
    x = torch.randn(T, W, generator=g).to(dtype)
    ids = torch.stack([torch.randperm(outputs, generator=g)[:top] for _ in range(T)]).to(torch.int32)
    z, place = ex.rows(x.cuda(), ids.cuda(), outputs)
    z, place = z.cpu().double(), place.cpu().long().view(T, top)
    assert sorted(place.flatten().tolist()) == list(range(T * top))
    up, down = ex.up.cpu().double(), ex.down.cpu().double()
    for t in range(T):
        for k in range(top):
            e = int(ids[t, k])
            if e < E:
                assert U.rel(z[place[t, k]], down[e] @ torch.relu(up[e] @ x[t].double()) ** 2) < bar


@pytest.mark.parametrize("M,N,K", [(1, 40, 64), (16, 100, 96), (5, 256, 1024), (40, 64, 96)])
def test_relu_square_product(M, N, K):
    from scratchpad_amd import _native
    g = torch.Generator().manual_seed(3)
    x, w = torch.randn(M, K, generator=g), torch.randn(N, K, generator=g) * K ** -0.5
    for dtype, bar in ((torch.float32, 2e-6), (torch.bfloat16, 1.2e-2)):
        got = _native.linear_relu_square(x.to(dtype).cuda(), w.to(dtype).cuda())
        assert U.rel(got, torch.relu(x.to(dtype).double() @ w.to(dtype).double().T) ** 2) < bar


# ------------------------------------------------------------------------------------------------ the attention kernels
class AttnBench:
    """the store + attention kernels as the model drives them, on shuffled slots of a NaN-filled pool"""

    def __init__(self, H, G, D, rot=None, dtype=torch.float32, matrix=True, scale=0.25, **kw):
        from scratchpad_amd.layers import HalfAngleRotary
        self.H, self.G, self.D, self.dtype, self.matrix, self.scale, self.kw = H, G, D, dtype, matrix, scale, kw
        self.rotary = HalfAngleRotary(rot["dims"], rot["base"]).cuda() if rot else None
        P = 700
        self.k = torch.full((P + 1, G * D), float("nan"), dtype=dtype, device="cuda")
        self.v = torch.full((P + 1, G * D), float("nan"), dtype=dtype, device="cuda")
        self.slots = (torch.randperm(P, generator=torch.Generator().manual_seed(9)) + 1).to(torch.int32).cuda()
        self.table = torch.zeros((4, P), dtype=torch.int32, device="cuda")
        self.table[2] = self.slots
        self.held = 0

    def step(self, q, k):
        from scratchpad_amd import _native as n_
        n = q.shape[0]
        loc = self.slots[self.held:self.held + n].long()
        pos = torch.arange(self.held, self.held + n, device="cuda")
        seq = seq_params(2, self.held, n)
        qk = torch.cat([q, k], 1).to(self.dtype).cuda()                    # views of one product, as in the model
        q, k = qk[:, :self.H * self.D], qk[:, self.H * self.D:]
        c = lambda name: None if self.kw.get(name) is None else self.kw[name].cuda()
        n_.qkv_rotary_store(q, k, None, self.k, self.v, pos, loc, self.rotary.freq if self.rotary else None, 1.0, self.H, self.G,
                            self.D, self.D, 1e-6, norm_values=False, q_bias=c("qb"), k_bias=c("kb"), qk_norm=2,
                            q_norm_weight=c("qn"), k_norm_weight=c("kn"))
        out = n_.window_attention(q, self.k, self.v, None, None, self.table, seq, self.H, self.G, self.D, self.D, 0, 0,
                                  self.scale, self.matrix)
        self.held += n
        return out.float().cpu()

    def run(self, q, k, sizes):
        return torch.cat([self.step(q[at:at + m], k[at:at + m]) for at, m in portions(q.shape[0], sizes)])


def attn_oracle(q, k, H, G, D, scale=0.25, rot=None, qb=None, kb=None, qn=None, kn=None):
    """the oracle's attention on ready projections: identity matrices stand for the products"""
    n, m = H * D, G * D
    eye = torch.eye(n + m, dtype=torch.float64)
    one = lambda t, size: torch.zeros(size, dtype=torch.float64) if t is None else t.double()
    w = {"a.q": eye[:n], "a.k": eye[n:], "a.q.b": one(qb, n), "a.k.b": one(kb, m),
         "a.q.norm": torch.ones(D, dtype=torch.float64) if qn is None else qn.double(),
         "a.k.norm": torch.ones(D, dtype=torch.float64) if kn is None else kn.double(), "a.o": eye[:n, :n]}
    spec = {"heads": H, "kv_heads": G, "dim": D, "vdim": D, "scale": scale}
    if rot:
        spec["rot"] = rot
    return mo.attention(torch.cat([q, k], 1).double(), w, "a", spec, 1e-6)


@pytest.mark.parametrize("sizes", [[150], [1], [7, 2, 40, 1, 1, 1, 3, 64, 1], [2]], ids=["whole", "decode", "mixed", "pairs"])
@pytest.mark.parametrize("shape", [(4, 2, 16, 8), (2, 2, 8, 8), (3, 1, 72, 10), (6, 3, 40, 0), (2, 1, 136, 64), (1, 1, 250, 250),
                                   (2, 1, 11, 4)], ids=lambda s: "x".join(map(str, s)))
def test_attention_on_keys_that_are_values(shape, sizes):
    """a bias, a weighted norm before the rotation, scores of several units: a key wrongly seen or missed, a norm after the
    rotation or without its weight, a value with norm, rotation or no bias each move the output by far more than the bar;
    every position of 150 is compared"""
    H, G, D, dims = shape
    g = torch.Generator().manual_seed(3)
    T = 150
    q, k = torch.randn(T, H * D, generator=g), torch.randn(T, G * D, generator=g)
    kw = dict(qb=torch.randn(H * D, generator=g), kb=torch.randn(G * D, generator=g), qn=1 + 0.5 * torch.randn(D, generator=g),
              kn=1 + 0.5 * torch.randn(D, generator=g))
    rot = {"dims": dims, "base": 100.0} if dims else None
    scale = 6.0 / D
    got = AttnBench(H, G, D, rot, scale=scale, **kw).run(q, k, sizes)
    want = attn_oracle(q, k, H, G, D, scale, rot, **kw)
    assert U.rel(got, want) < 2e-5
    for drop in kw:                                                       # the oracle moves when a piece is left out
        assert U.rel(attn_oracle(q, k, H, G, D, scale, rot, **{**kw, drop: None}), want) > 1e-2, drop


@pytest.mark.parametrize("D", [16, 64])
def test_far_key_and_a_tempting_future_key(D):
    """one key at position 3 among 600 whose score stands out: every later query hears its value, in a prompt of 600 and
    decoded token by token behind a prompt; a key that would win at position p + 1 must never reach query p"""
    T = 600
    g = torch.Generator().manual_seed(1)
    q, k = torch.randn(T, D, generator=g) * 0.1, torch.randn(T, D, generator=g) * 0.1
    q[:, 0], k[:, 1] = 6.0, 1.0
    k[3] = 0.1 * torch.linspace(-1, 1, D)
    k[3, 0], k[3, 2] = 40.0, 20.0                              # normed: a cosine of 0.89 to coordinate 0, against 0.1 of the others
    k[400] = 0.1 * torch.linspace(1, -1, D)
    k[400, 0] = 90.0                                           # position 399 must not see it; 400 and later do
    kn = torch.full((D,), 3.0)
    scale = 10.0 / D                                           # the best score is about 30
    want = attn_oracle(q, k, 1, 1, D, scale, kn=kn)
    cos = lambda a, b: float(torch.dot(a.double(), b.double()) / a.double().norm() / b.double().norm())
    assert cos(want[399], k[3]) > 0.999 and cos(want[2], k[3]) < 0.9 and float(want[400, 0]) > 80
    for dtype, bar in ((torch.float32, 2e-5), (torch.bfloat16, 2e-2)):
        for sizes in ([T], [390, 1], [64], [63, 2, 1]):
            got = AttnBench(1, 1, D, dtype=dtype, scale=scale, kn=kn).run(q, k, sizes)
            assert cos(got[399], k[3]) > 0.999 and cos(got[150], k[3]) > 0.999 and float(got[399, 0]) < 45
            assert U.rel(got, want) < bar


@pytest.mark.parametrize("sizes", [[200], [17, 2, 64, 1, 1, 33, 16, 5], [3]], ids=["whole", "mixed", "threes"])
@pytest.mark.parametrize("shape", [(8, 2, 128), (4, 4, 64), (6, 1, 128)], ids=lambda s: "x".join(map(str, s)))
def test_matrix_core_attention_against_the_vector_kernel(shape, sizes):
    """portions of prompts in bf16 with heads of 64 / 128 run on the matrix cores: against the fp32-arithmetic vector kernel
    that the tests above pin (same cache, same portions)"""
    H, G, D = shape
    g = torch.Generator().manual_seed(7)
    q, k = torch.randn(200, H * D, generator=g), torch.randn(200, G * D, generator=g)
    kw = dict(qn=1 + 0.3 * torch.randn(D, generator=g), kn=1 + 0.3 * torch.randn(D, generator=g), kb=torch.randn(G * D, generator=g))
    outs = [AttnBench(H, G, D, {"dims": D // 2, "base": 1000.0}, dtype=torch.bfloat16, matrix=m, scale=4.0 / D, **kw).run(q, k, sizes)
            for m in (True, False)]
    assert torch.isfinite(outs[0]).all()
    assert U.rel(outs[0], outs[1]) < 1.5e-2


# ------------------------------------------------------------------------------------------------ the whole model
@pytest.fixture(scope="module")
def full(tmp_path_factory):
    cfg = U.full_config()
    folder, w = U.make_model(tmp_path_factory.mktemp("full"), cfg, seed=11)
    toks = U.tokens(130, cfg["vocab"], 12)
    lay = []
    want = mo.forward(toks, w, cfg, lay)
    return cfg, folder, w, toks, want, lay


def test_whole_prompt_with_the_stream_after_every_layer(full):
    cfg, folder, w, toks, want, lay = full
    eng = engine(folder)
    eng.runner.model.capture_layers = []
    got = run_whole(eng, toks)
    assert len(eng.runner.model.capture_layers) == len(cfg["layers"])
    for i, (a, b) in enumerate(zip(eng.runner.model.capture_layers, lay)):
        assert U.rel(a, b) < F32_BAR, i
    assert U.rel(got, want) < F32_BAR
    eng.runner.model.capture_layers = None
    assert U.rel(run_whole(eng, toks, "again"), want) < F32_BAR            # on rows and slots used before


def test_serving_precision(full):
    cfg, folder, w, toks, want, _ = full
    for sizes in ([130], [60, 1]):
        got = run_portions(engine(folder, dtype=torch.bfloat16), toks, sizes)
        err = (got.double().cpu() - want).abs().amax(-1) / want.abs().max()
        # (a router's close call that falls the other way in 16 bits moves single positions by more: the bulk is the bar)
        assert float(err.median()) < 5e-2 and float(err.quantile(0.9)) < 0.15


@pytest.mark.parametrize("graphs", [False, True], ids=["eager", "graphs"])
def test_decoding_from_the_first_token(full, graphs):
    """130 single-token steps: the first is a first token on a fresh slot, every later one a decode step through the cache"""
    cfg, folder, w, toks, want, _ = full
    assert U.rel(run_portions(engine(folder, graphs=graphs), toks, [1]), want) < F32_BAR


def test_long_decoding_behind_a_prompt(tmp_path):
    cfg = U.config([(U.attention(2, 1, 16), U.moe(4, 2, 24, identity=2, count=2, keep=1, shared=16)), 0], width=48, vocab=61)
    folder, w = U.make_model(tmp_path, cfg, seed=8)
    toks = U.tokens(400, 61, 9)
    want = mo.forward(toks, w, cfg)
    assert U.rel(run_portions(engine(folder, graphs=True), toks, [40, 1]), want) < F32_BAR


@pytest.mark.parametrize("sizes", [[2], [3, 2, 17, 1, 1, 64, 5, 1], [64, 2, 1], [15, 16, 17, 1]],
                         ids=["pairs", "mixed", "big-then-small", "near-16"])
def test_portions_of_prompts(full, sizes):
    cfg, folder, w, toks, want, _ = full
    assert U.rel(run_portions(engine(folder), toks, sizes), want) < F32_BAR


def test_garbage_in_reused_slots_is_never_read(full):
    cfg, folder, w, toks, want, _ = full
    eng = engine(folder)
    for b in eng.runner.token_to_kv_pool._all():
        b.fill_(float("nan"))
    assert U.rel(run_portions(eng, toks[:60], [7, 1]), want[:60]) < F32_BAR


def test_borrowed_tensors_keep_a_cache_per_layer(tmp_path):
    """the same tensors three times in a row: every run has rows of its own in the pool (they differ), and wiping one run's
    rows between two steps changes what follows"""
    cfg = U.config([(U.attention(2, 1, 16), None), 0, 1], width=48)
    folder, w = U.make_model(tmp_path, cfg, seed=3)
    toks = U.tokens(30, cfg["vocab"], 2)
    want = mo.forward(toks, w, cfg)
    eng = engine(folder)
    first = eng.step([entry("a", toks[:20])])
    pool = eng.runner.token_to_kv_pool
    k = [pool.get_key_buffer(i) for i in range(3)]
    assert not torch.equal(k[0], k[1]) and not torch.equal(k[1], k[2])
    second = eng.step([entry("a", toks[20:25])])
    assert U.rel(torch.cat([first, second]), want[:25]) < F32_BAR
    pool.get_value_buffer(1).zero_()
    assert U.rel(eng.step([entry("a", toks[25:])], ["a"]), want[25:]) > 1e-2


@pytest.mark.parametrize("graphs", [False, True], ids=["eager", "graphs"])
def test_unequal_batches_with_rows_and_slots_reused(full, graphs):
    """seven requests of unequal length through three rows and a pool that holds far fewer tokens than their sum: portions
    of some beside single tokens of others, pauses, rows and slots handed on; every request's logits must be what it gets
    alone"""
    cfg, folder, w, _, _, _ = full
    reqs = {f"r{i}": U.tokens(n, cfg["vocab"], 20 + i) for i, n in enumerate([45, 3, 70, 1, 26, 58, 12])}
    want = {r: mo.forward(t, w, cfg) for r, t in reqs.items()}
    eng = engine(folder, tokens=200, slots=3, graphs=graphs)
    plan = {"r0": [5, 1, 1, 30, 1, 7], "r1": [2, 1], "r2": [33, 2, 1, 1, 1, 1, 1, 30], "r3": [1], "r4": [1, 1, 24],
            "r5": [2, 50, 1, 1, 1, 1, 1, 1], "r6": [6, 1, 1, 1, 1, 1, 1]}
    fed, got, waiting, live, step = {r: 0 for r in reqs}, {r: [] for r in reqs}, list(reqs), [], 0
    while waiting or live:
        while waiting and len(live) < 3 and sum(len(reqs[r]) for r in live) + len(reqs[waiting[0]]) <= 200:
            live.append(waiting.pop(0))
        entries, end = [], []
        for r in live:
            if (step + int(r[1:])) % 5 == 4 and len(live) > 1:
                continue                                           # left out of this step, goes on later
            n = min(plan[r].pop(0) if plan[r] else 1, len(reqs[r]) - fed[r])
            entries.append(entry(r, reqs[r][fed[r]:fed[r] + n]))
            fed[r] += n
            if fed[r] == len(reqs[r]):
                end.append(r)
        if entries:
            out = eng.step(entries, end)
            at = 0
            for e in entries:
                got[e.rid].append(out[at:at + len(e.tokens)])
                at += len(e.tokens)
        live = [r for r in live if r not in end]
        step += 1
    for r in reqs:
        assert U.rel(torch.cat(got[r]), want[r]) < F32_BAR, r


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["fp32", "bf16"])
def test_graph_replay_of_larger_decode_steps(full, dtype):
    """40 requests decoding together; every replay (six, with eager steps of the other engine and synchronisations between)
    is compared with the same step run eagerly"""
    cfg, folder, w, _, _, _ = full
    reqs = {f"q{i}": U.tokens(3 + i % 9, cfg["vocab"], 300 + i) + U.tokens(6, cfg["vocab"], 900 + i) for i in range(40)}
    engines = [engine(folder, dtype=dtype, tokens=900, slots=40, graphs=graphs) for graphs in (True, False)]
    for eng in engines:
        eng.step([entry(r, t[:-6], []) for r, t in reqs.items()])                     # the prompts, one extend batch
    outs = [[], []]
    for k in range(6):
        for eng, steps in zip(engines, outs):
            steps.append(eng.step([entry(r, [t[len(t) - 6 + k]]) for r, t in reqs.items()], list(reqs) if k == 5 else []))
            torch.cuda.synchronize()
    outs = [torch.stack(s) for s in outs]
    bar = 1e-5 if dtype == torch.float32 else 3e-2
    for k in range(6):
        assert U.rel(outs[0][k], outs[1][k]) < bar, k
    if dtype == torch.float32:
        want = torch.stack([mo.forward(t, w, cfg)[-6:] for t in reqs.values()], 1)    # [step, request, vocab]
        assert U.rel(outs[0], want) < F32_BAR


def test_generation_through_the_scheduler(full):
    """greedy generation of three prompts through Engine.generate (admission, chunked prefill of 16 tokens beside decoding
    requests, release) equals the oracle's greedy continuation; sampled generation runs and stays in the vocabulary"""
    from scratchpad_amd.sampler import SamplingParams
    cfg, folder, w, _, _, _ = full
    prompts = [U.tokens(n, cfg["vocab"], 40 + n) for n in (37, 5, 21)]
    eng = engine(folder, tokens=300, slots=2, graphs=True, chunk=16)
    got = eng.generate(prompts, max_new_tokens=12)
    for p, out in zip(prompts, got):
        ref = U.greedy(p, w, cfg, 12)
        agree = next((i for i, (a, b) in enumerate(zip(out, ref)) if a != b), 12)
        if agree < 12:      # a near-tie in fp32 against float64 may flip one choice: the logits there must be that close
            lg = mo.forward(p + ref[:agree], w, cfg)[-1]
            assert float(lg[ref[agree]] - lg[out[agree]]) < 1e-3 * float(lg.abs().max()), (agree, out, ref)
        else:
            assert out == ref
    sampled = eng.generate(prompts[:2], SamplingParams(max_new_tokens=6, temperature=0.8, top_p=0.9, top_k=20))
    assert all(len(o) == 6 and all(0 <= t < cfg["vocab"] for t in o) for o in sampled)


@pytest.mark.parametrize("seed", range(10))
def test_designs_drawn_at_random(tmp_path, seed):
    """layer order, borrowed tensors, sizes and constants drawn at random: whole prompt, then portions of random sizes with
    single tokens between them, both against the oracle"""
    import random
    cfg = U.random_config(100 + seed)
    folder, w = U.make_model(tmp_path, cfg, seed=seed)
    toks = U.tokens(90, cfg["vocab"], seed)
    want = mo.forward(toks, w, cfg)
    assert U.rel(run_whole(engine(folder), toks), want) < F32_BAR, cfg
    r = random.Random(seed)
    sizes = [r.choice([1, 1, 2, 3, 7, 16, 29]) for _ in range(40)]
    assert U.rel(run_portions(engine(folder), toks, sizes), want) < F32_BAR, (sizes, cfg)


def test_sizes_that_are_one_or_equal(tmp_path):
    """a model whose sizes are 1 or equal where the others' differ: one head, head width = model width, rotation over the
    whole head, alpha and scale 1, one expert that is always chosen, then one identity expert beside one expert"""
    cfg = U.config([
        (U.attention(1, 1, 16, dims=16, scale=1.0), U.moe(1, 1, 16, shared=16)),
        (U.attention(1, 1, 16, dims=2, scale=1.0), U.moe(1, 1, 16, identity=1)),
        (U.attention(16, 16, 16, dims=16, scale=1.0), U.moe(1, 2, 16, identity=1, count=2, keep=2)),
        0,
    ], width=16, vocab=17, alpha=1.0)
    folder, w = U.make_model(tmp_path, cfg, seed=4)
    toks = U.tokens(50, 17, 3)
    want = mo.forward(toks, w, cfg)
    assert U.rel(run_whole(engine(folder), toks), want) < F32_BAR
    assert U.rel(run_portions(engine(folder), toks, [3, 1]), want) < F32_BAR
