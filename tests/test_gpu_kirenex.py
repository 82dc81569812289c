"""Kirenex through the engine on the GPU against the CPU oracle (float64, one sequence at a time, no cache or state): single
mechanisms, kernels on crafted inputs (a far key among hundreds, tempting keys one position outside a window and one ahead, kept
first tokens, decays that keep the first token audible), whole prompts with the stream after every layer, decoding through
caches and states, portions down to two tokens, unequal batches, reused rows and slots, graph replay, other sizes, and
generation through the engine's scheduler.

Sharp comparisons run the engine in fp32 (the oracle's weights are bf16-representable, so both see the same numbers); a
bf16 pass checks the serving precision against a looser bar."""
import math

import pytest
import torch

from oracle import kirenex as ko
from tests import kirenex_util as U
from tests.test_gpu_toredra import engine, entry, portions, run_portions, run_whole, seq_params

pytestmark = pytest.mark.gpu
F32_BAR = 2e-4
CUTS = {"whole": [150], "decode": [1], "mixed": [7, 2, 40, 1, 1, 1, 3, 64, 1], "pairs": [2]}


# ------------------------------------------------------------------------------------------------ mechanisms alone
LAYERS = [
    [(U.latent(4, 16, 8, 24, 40), None)],
    [(U.latent(3, 24, 12, 8, 72, base=20.0), U.dense(40))],
    [(U.latent(1, 8, 2, 8, 8), None)],                                      # one head, one rotated pair
    [(U.latent(17, 8, 24, 16, 136, scale=0.3), None)],                      # more heads than a tile, more rotated than plain
    [(U.latent(2, 136, 64, 200, 264), U.dense(24))],
    [(U.latent(2, 16, 8, 24, 40), None), (U.latent(5, 24, 8, 16, 40, kv_from=0), U.dense(24))],
    [(U.parallel(4, 2, 16, 24, 4, 2, 8, 40, conv=4), None)],
    [(U.parallel(3, 3, 24, 8, 1, 1, 72, 8, size=5, keep=0, conv=2), U.dense(64))],        # nothing kept, kv heads = heads
    [(U.parallel(5, 1, 8, 72, 6, 3, 16, 16, size=1, keep=4, dims=0, conv=1), None)],      # a window of one, no rotation, one tap
    [(U.parallel(2, 1, 40, 16, 2, 1, 136, 136, size=24, keep=30, dims=20, scaling=False, conv=3), None)],   # more kept than the window
    [(U.parallel(2, 2, 136, 200, 2, 2, 24, 200, size=None, scale=0.02, conv=5), None)],   # plain causal, heads above 128
    [(U.parallel(2, 1, 16, 16, 3, 3, 20, 12, size=200, keep=3), U.dense(8))],             # a window longer than the prompt
]


@pytest.mark.parametrize("layers", LAYERS, ids=lambda l: "+".join(s["type"][:6] for s, _ in l))
@pytest.mark.parametrize("width", [80, 77])
def test_small_models_match_oracle(tmp_path, layers, width):
    cfg = U.config(layers, width=width)
    folder, w = U.make_model(tmp_path, cfg, seed=5)
    toks = U.tokens(70, cfg["vocab"], 6)
    eng = engine(folder)
    eng.runner.model.capture_layers = []
    got = run_whole(eng, toks)
    lay = []
    want = ko.forward(toks, w, cfg, lay)
    for a, b in zip(eng.runner.model.capture_layers, lay):
        assert U.rel(a, b) < F32_BAR
    assert U.rel(got, want) < F32_BAR


# ------------------------------------------------------------------------------------------------ row kernels
@pytest.mark.parametrize("W", [200, 77, 96, 3000, 4100])
def test_post_norm_of_two_branches(W):
    from scratchpad_amd import _native
    g = torch.Generator().manual_seed(0)
    T, eps, alpha = 37, 1e-5, 2.5
    rn = lambda *s: torch.randn(*s, generator=g)
    x, a, b = rn(T, W) * torch.linspace(0.1, 9.0, W), rn(T, 2 * W) * 3, rn(T, W) * 0.02
    wa, wb, w = (1 + 0.3 * rn(W) for _ in range(3))
    for dtype, bar in ((torch.float32, 2e-6), (torch.bfloat16, 1e-2)):
        for want_lo in (True, False):
            av, bv = a.to(dtype).cuda()[:, W:], b.to(dtype).cuda()                         # a view: its stride is taken
            y = ko.average_of_normed(av.double().cpu(), bv.double().cpu(), wa.double(), wb.double(), eps)
            want = ko.post_norm(x.double(), y, w.double(), alpha, eps)
            xs = x.clone().cuda()
            lo = _native.post_norm(xs, av, w.cuda(), eps, alpha, dtype, b=bv, wa=wa.cuda(), wb=wb.cuda(), want_lo=want_lo)
            assert U.rel(xs, want) < 2e-6
            assert (lo is None) != want_lo and (lo is None or (lo.dtype == dtype and U.rel(lo, want) < bar))


def test_embedding_with_positions():
    from scratchpad_amd import _native
    g = torch.Generator().manual_seed(1)
    for W in (96, 77):
        for dtype in (torch.float32, torch.bfloat16):
            emb, table = torch.randn(50, W, generator=g).to(dtype).cuda(), torch.randn(30, W, generator=g).to(dtype).cuda()
            ids, pos = torch.randint(0, 50, (40,), generator=g).cuda(), torch.randint(0, 30, (40,), generator=g).cuda()
            x, lo = _native.embed_scale(emb, ids, 1.0, want_lo=True, table=table, positions=pos)
            want = emb[ids].float() + table[pos].float()
            assert torch.equal(x, want) and torch.equal(lo, want.to(dtype))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16, torch.float16])
def test_gelu_products_agree_with_torch_and_with_each_other(dtype):
    """the activation alone, and behind the weight-streaming product of a few rows - which is the same two steps bit for bit"""
    from scratchpad_amd import _native
    g = torch.Generator().manual_seed(2)
    for T, d in ((5, 64), (300, 41), (1, 2048)):
        x = (torch.randn(T, 2 * d, generator=g) * 3).to(dtype).cuda()
        want = torch.nn.functional.gelu(x[:, :d].double(), approximate="tanh") * x[:, d:].double()
        assert U.rel(_native.gelu_tanh_and_mul(x), want.cpu()) < (1e-6 if dtype == torch.float32 else 5e-3)
    for T, K, ff in ((1, 64, 48), (8, 2048, 128), (5, 96, 24), (40, 96, 24)):
        h, w = torch.randn(T, K, generator=g).to(dtype).cuda(), (torch.randn(2 * ff, K, generator=g) * K ** -0.5).to(dtype).cuda()
        want = ko.gelu_tanh(h.double().cpu() @ w[:ff].double().cpu().T) * (h.double().cpu() @ w[ff:].double().cpu().T)
        got = _native.linear_gelu_mul(h, w)
        assert U.rel(got, want) < (1e-5 if dtype == torch.float32 else 2e-2)
        if dtype != torch.float32 and T <= 8:
            fused = _native._skinny_glu(h, w, False, 3, "test")
            plain = torch.empty(T, 2 * ff, dtype=dtype, device="cuda")
            _native._check(_native.load().sp_gemm_skinny(plain.data_ptr(), h.data_ptr(), w.data_ptr(), T, 2 * ff, K, K, K, 2 * ff, 0,
                                                         _native._dt(h), _native._stream()), "test")
            assert fused is not None and torch.equal(fused, _native.gelu_tanh_and_mul(plain)) and torch.equal(fused, got)


@pytest.mark.parametrize("H,K,N,T", [(3, 24, 72, 40), (1, 8, 8, 1), (5, 12, 10, 70), (2, 136, 264, 9), (4, 64, 40, 300), (16, 32, 128, 65)])
def test_head_linear(H, K, N, T):
    """a product per head on views of a larger row, with and without the output gate; 65 and more tokens take the wide tiles"""
    from scratchpad_amd import _native
    g = torch.Generator().manual_seed(3)
    row, w = torch.randn(T, H * (K + 16) + H * N, generator=g), torch.randn(H, N, K, generator=g) * K ** -0.5
    for dtype, bar in ((torch.float32, 1e-5), (torch.bfloat16, 1e-2)):
        a, ww = row.to(dtype).cuda(), w.to(dtype).cuda()
        x = a[:, :H * (K + 16)].view(T, H, K + 16)[:, :, :K]
        gate = a[:, H * (K + 16):]
        want = torch.einsum("thk,hnk->thn", x.double().cpu(), ww.double().cpu())
        assert U.rel(_native.head_linear(x, ww), want) < bar
        want = want * torch.sigmoid(gate.double().cpu()).view(T, H, N)
        assert U.rel(_native.head_linear(x, ww, gate=gate), want) < bar


# ------------------------------------------------------------------------------------------------ short convolution
def many_requests(held, lens, rows):
    from scratchpad_amd import _native
    dev = "cuda"
    i32 = lambda x: torch.tensor(x, dtype=torch.int32, device=dev)
    start = [sum(lens[:i]) for i in range(len(lens))]
    return _native.SeqParams(torch.tensor(rows, device=dev), torch.tensor([h + n for h, n in zip(held, lens)], device=dev), i32(lens),
                             i32(held), i32(start), torch.repeat_interleave(torch.arange(len(lens), dtype=torch.int32, device=dev),
                                                                            torch.tensor(lens, device=dev)))


@pytest.mark.parametrize("taps", [1, 2, 3, 4, 5])
@pytest.mark.parametrize("C", [64, 72, 52], ids=["pieces", "pieces-odd", "fp32-pieces"])
def test_convolution_across_portions_and_requests(taps, C):
    """three requests interleaved in steps of unequal portions (more than 64 rows: a row read once for all taps; fewer: the plain
    form; single tokens: output and state in one launch), from NaN-filled state rows"""
    from scratchpad_amd import _native
    g = torch.Generator().manual_seed(taps)
    T, rows = 97, [4, 1, 6]
    w = torch.randn(C, taps, generator=g)
    for dtype, bar in ((torch.float32, 2e-6), (torch.bfloat16, 1e-2)):
        u = [torch.randn(T, 2 * C, generator=g).to(dtype) for _ in rows]
        want = [ko.silu(ko.causal_conv(x[:, C:].double(), w.double())) for x in u]
        state = torch.full((8, max(taps - 1, 0), C), float("nan"), device="cuda")
        held, got = [0, 0, 0], [[], [], []]
        for step in ([40, 1, 33], [1, 1, 1], [1, 30, 2], [20, 50, 1], [1, 1, 1], [1, 1, 1], [33, 13, 58]):
            assert all(h + n <= T for h, n in zip(held, step))
            x = torch.cat([u[i][held[i]:held[i] + n, C:] for i, n in enumerate(step)])
            wide = torch.zeros(x.shape[0], 2 * C, dtype=dtype)
            wide[:, C:] = x
            if all(n == 1 for n in step) and all(h > 0 for h in held):
                seq = _native.SeqParams(torch.tensor(rows, device="cuda"), torch.tensor([h + 1 for h in held], device="cuda"))
            else:
                seq = many_requests(held, step, rows)
            out = _native.causal_conv_silu(wide.cuda()[:, C:], w.cuda(), None, state, seq).cpu()
            at = 0
            for i, n in enumerate(step):
                got[i].append(out[at:at + n])
                at, held[i] = at + n, held[i] + n
        for i in range(3):
            assert U.rel(torch.cat(got[i]), want[i][:held[i]]) < bar, (i, dtype)
        if taps > 1:
            assert torch.isnan(state[0]).all() and torch.isnan(state[7]).all()             # neighbouring rows untouched


# ------------------------------------------------------------------------------------------------ the delta rule's kernel
def delta_inputs(T, H, G, D, Dv):
    """decays of 0.99 and more in most heads: what token 0 wrote (in full, later ones lightly) is still read at the end"""
    g = torch.Generator().manual_seed(4)
    q, k, v, gate = (torch.randn(T, n, generator=g) for n in (G * D, G * D, H * Dv, H * Dv))
    pre = torch.cat([torch.randn(T, H, generator=g) - 4.0, torch.randn(T, H, generator=g) - 3.0], 1)
    pre[0, :H] = 4.0
    A, dt = torch.full((H,), -3.0), torch.randn(H, generator=g) * 0.3
    if H > 1:
        A[H // 2] = 0.5                                                    # one head forgets fast: heads are not alike
    return q, k, v, gate, pre, A, dt, 1 + 0.3 * torch.randn(Dv, generator=g)


def delta_oracle(q, k, v, gate, pre, A, dt, nw, H, G, D, Dv, eps):
    T, r = q.shape[0], H // G
    q, k, v = ko.unit(q.double().view(T, G, D)) * D ** -0.5, ko.unit(k.double().view(T, G, D)), v.double().view(T, H, Dv)
    beta = torch.sigmoid(pre[:, :H].double())
    decay = torch.exp(-torch.exp(A.double()) * ko.softplus(pre[:, H:].double() + dt.double()))
    o = torch.stack([ko.delta_scan(q[:, h // r], k[:, h // r], v[:, h], beta[:, h], decay[:, h]) for h in range(H)], 1)
    return (ko.rms(o, eps) * nw.double() * ko.silu(gate.double()).view(T, H, Dv)).reshape(T, H * Dv)


@pytest.mark.parametrize("cut", CUTS)
@pytest.mark.parametrize("shape", [(4, 2, 16, 24), (2, 2, 32, 64), (3, 1, 8, 200), (2, 1, 136, 40), (1, 1, 64, 136), (6, 3, 72, 16),
                                   (2, 1, 20, 12), (1, 1, 5, 3), (2, 2, 128, 128), (1, 1, 256, 256)], ids=lambda s: "x".join(map(str, s)))
def test_head_delta_scan_keeps_the_first_token_audible(shape, cut):
    from scratchpad_amd import _native
    H, G, D, Dv = shape
    T, eps = 150, 1e-5
    x = delta_inputs(T, H, G, D, Dv)
    want = delta_oracle(*x, H, G, D, Dv, eps)
    late = delta_oracle(*[t[1:] for t in x[:5]], *x[5:], H, G, D, Dv, eps)
    assert U.rel(late[-1], want[-1]) > 1e-3                               # token 0 is audible at the end
    c = lambda t: t.cuda()
    for ranges in (None, 1, 3):
        state = torch.full((4, H, D, Dv), float("nan"), device="cuda")
        outs, held = [], 0
        for at, n in portions(T, CUTS[cut]):
            s = slice(at, at + n)
            outs.append(_native.head_delta_scan(*[c(t[s]) for t in x[:5]], c(x[6]), c(x[5]), c(x[7]), state, seq_params(2, held, n), H, G,
                                                D, Dv, eps, ranges=ranges).cpu())
            held += n
        assert U.rel(torch.cat(outs), want) < 2e-5, ranges
        assert torch.isnan(state[1]).all() and torch.isnan(state[3]).all()     # neighbouring slots untouched


def test_head_delta_scan_of_several_requests_in_one_step():
    from scratchpad_amd import _native
    H, G, D, Dv, eps = 4, 2, 24, 40, 1e-5
    lens, rows = [33, 1, 16, 17], [5, 2, 7, 1]
    x = [delta_inputs(n + 20, H, G, D, Dv) for n in lens]
    c = lambda t: t.cuda()
    for dtype, bar in ((torch.float32, 2e-5), (torch.bfloat16, 2e-2)):
        state = torch.full((9, H, D, Dv), float("nan"), device="cuda")
        got = [[] for _ in lens]
        for held, step in (([0] * 4, lens), (lens, [20] * 4)):
            cat = [torch.cat([xi[j][h:h + n] for xi, h, n in zip(x, held, step)]) for j in range(5)]
            low = [t.to(dtype) for t in cat[:4]]
            out = _native.head_delta_scan(*map(c, low), c(cat[4]), c(x[0][6]), c(x[0][5]), c(x[0][7]), state,
                                          many_requests(held, step, rows), H, G, D, Dv, eps).float().cpu()
            at = 0
            for i, n in enumerate(step):
                got[i].append(out[at:at + n])
                at += n
        for i, xi in enumerate(x):
            low = [t.to(dtype).float() for t in xi[:4]]
            assert U.rel(torch.cat(got[i]), delta_oracle(*low, xi[4], *x[0][5:], H, G, D, Dv, eps)) < bar, i


# ------------------------------------------------------------------------------------------------ latent attention's kernels
class LatentBench:
    """store + attention as the model drives them, on shuffled slots of a NaN-filled pool"""

    def __init__(self, H, D, R, C, dtype=torch.float32, scale=0.2, base=100.0, **kw):
        from scratchpad_amd.layers import AngleRotary
        self.H, self.D, self.R, self.C, self.dtype, self.scale, self.kw = H, D, R, C, dtype, scale, kw
        self.rot = {"dims": R, "base": base}
        self.rotary = AngleRotary(R, base).cuda()
        P = 700
        self.pool = torch.full((P + 1, C + R), float("nan"), dtype=dtype, device="cuda")
        self.slots = (torch.randperm(P, generator=torch.Generator().manual_seed(9)) + 1).to(torch.int32).cuda()
        self.table = torch.zeros((4, P), dtype=torch.int32, device="cuda")
        self.table[2] = self.slots
        self.held = 0

    def run(self, dkv, q, q_lat, nw, sizes):
        from scratchpad_amd import _native as n_
        outs = []
        for at, n in portions(dkv.shape[0], sizes):
            c = lambda t: t[at:at + n].to(self.dtype).cuda()
            loc, pos = self.slots[self.held:self.held + n].long(), torch.arange(self.held, self.held + n, device="cuda")
            qq = c(q).view(n, self.H, self.D + self.R)
            n_.latent_kv_store(self.pool, c(dkv), nw.cuda(), pos, self.rotary.freq, 1.0, loc, self.C, 1e-5, q=qq, q_offset=self.D)
            outs.append(n_.latent_attention(c(q_lat), qq[:, :, self.D:], self.pool, self.table, seq_params(2, self.held, n), self.scale,
                                            token_major=True, **self.kw).float().cpu())
            self.held += n
        return torch.cat(outs)

    def oracle(self, dkv, q, q_lat, nw):
        T, r = dkv.shape[0], lambda t: t.to(self.dtype).double()
        c = ko.rms(r(dkv)[:, :self.C], 1e-5) * nw.double()
        kr = ko.rotate_neighbours(r(dkv)[:, None, self.C:], self.rot)[:, 0]
        qr = ko.rotate_neighbours(r(q).view(T, self.H, self.D + self.R)[..., self.D:], self.rot)
        s = torch.stack([r(q_lat)[:, h] @ c.T + qr[:, h] @ kr.T for h in range(self.H)], 1) * self.scale
        seen = torch.ones(T, T, dtype=torch.bool).tril()[:, None]
        return torch.softmax(s.masked_fill(~seen, -math.inf), -1) @ c


def latent_inputs(T, H, D, R, C, seed=3):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(T, C + R, generator=g), torch.randn(T, H * (D + R), generator=g), torch.randn(T, H, C, generator=g) * 2,
            1 + 0.3 * torch.randn(C, generator=g))


@pytest.mark.parametrize("cut", CUTS)
@pytest.mark.parametrize("shape", [(3, 16, 8, 40), (1, 8, 2, 8), (5, 24, 12, 72), (18, 8, 16, 24), (2, 16, 24, 136), (4, 40, 64, 264)],
                         ids=lambda s: "x".join(map(str, s)))
def test_latent_attention_in_fp32(shape, cut):
    H, D, R, C = shape
    x = latent_inputs(150, H, D, R, C)
    b = LatentBench(H, D, R, C, scale=2.0 / C)
    got = b.run(*x, CUTS[cut])
    assert U.rel(got, b.oracle(*x)) < 2e-5


@pytest.mark.parametrize("cut", CUTS)
@pytest.mark.parametrize("H,R,C", [(3, 8, 40), (16, 16, 96), (5, 32, 128), (20, 8, 200), (33, 64, 256), (2, 64, 136), (16, 64, 512),
                                   (40, 8, 504), (7, 56, 264), (70, 16, 72)], ids=lambda v: str(v))
def test_latent_attention_on_the_matrix_cores(H, R, C, cut):
    """every tile shape (row widths up to 160, 320, 576; row blocks of 16, 32, 64 for single tokens and portions), keys shared out
    over 1 and 3 workgroups and as the step's size says, against the oracle on the same 16-bit inputs and against the vector kernel"""
    T, D = 150, 8
    x = latent_inputs(T, H, D, R, C)
    want = None
    for kw in (dict(splits=1), dict(splits=3), dict(), dict(matrix=False)):
        b = LatentBench(H, D, R, C, dtype=torch.bfloat16, scale=2.0 / C, **kw)
        if want is None:
            want = b.oracle(*x)
        got = b.run(*x, CUTS[cut])
        assert torch.isfinite(got).all() and U.rel(got, want) < 1.2e-2, kw


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["fp32", "bf16"])
def test_far_latent_key_and_a_tempting_future_key(dtype):
    """one loud key at position 3 among 600: every later query hears it, whole and decoded behind a prompt; a louder one at
    position 400 must not reach query 399, which is computed in the same tile"""
    H, D, R, C, T = 2, 8, 8, 64, 600
    dkv, q, q_lat, nw = latent_inputs(T, H, D, R, C, seed=1)
    nw = torch.ones(C)
    dkv[:, C:], q[:] = 0.0, 0.0                                           # the latent part alone decides
    q_lat *= 0.05
    q_lat[:, :, 0] = 8.0
    dkv[:, 0] = 0.0
    dkv[3] = 0.0
    dkv[3, 0], dkv[3, 5] = 4.0, 3.0
    dkv[400] = 0.0
    dkv[400, 0], dkv[400, 9] = 40.0, 10.0
    loud3, loud400 = (ko.rms(dkv[i:i + 1, :C].double(), 1e-5)[0] for i in (3, 400))
    cos = lambda a, z: float(torch.dot(a.double(), z) / a.double().norm() / z.norm())
    for sizes in ([T], [390, 1], [64], [63, 2, 1]):
        b = LatentBench(H, D, R, C, dtype=dtype, scale=0.5)
        got = b.run(dkv, q, q_lat, nw, sizes)
        want = b.oracle(dkv, q, q_lat, nw)
        assert cos(want[399, 0], loud3) > 0.99 and cos(want[400, 0], loud400) > 0.99 and cos(want[2, 0], loud3) < 0.5
        assert cos(got[399, 1], loud3) > 0.99 and cos(got[150, 0], loud3) > 0.99 and cos(got[400, 1], loud400) > 0.99
        assert U.rel(got, want) < (2e-5 if dtype == torch.float32 else 1.2e-2)


# ------------------------------------------------------------------------------------------------ windowed attention's kernels
class WindowBench:
    """the store + attention kernels as the model drives them, on shuffled slots of a NaN-filled pool"""

    def __init__(self, H, G, D, Dv, size, keep, rot=None, dtype=torch.float32, matrix=True, scale=0.25):
        from scratchpad_amd.layers import HalfAngleRotary
        self.H, self.G, self.D, self.Dv, self.size, self.keep, self.rot = H, G, D, Dv, size, keep, rot
        self.dtype, self.matrix, self.scale = dtype, matrix, scale
        self.rotary = HalfAngleRotary(rot["dims"], rot["base"], rot.get("scaling")).cuda() if rot else None
        P = 700
        self.k = torch.full((P + 1, G * D), float("nan"), dtype=dtype, device="cuda")
        self.v = torch.full((P + 1, G * Dv), float("nan"), dtype=dtype, device="cuda")
        self.slots = (torch.randperm(P, generator=torch.Generator().manual_seed(9)) + 1).to(torch.int32).cuda()
        self.table = torch.zeros((4, P), dtype=torch.int32, device="cuda")
        self.table[2] = self.slots
        self.held = 0

    def run(self, q, k, v, qw, kw, sizes):
        from scratchpad_amd import _native as n_
        outs = []
        for at, n in portions(q.shape[0], sizes):
            c = lambda t: t[at:at + n].to(self.dtype).cuda()
            loc, pos = self.slots[self.held:self.held + n].long(), torch.arange(self.held, self.held + n, device="cuda")
            qq = c(q)
            freq, mag = (self.rotary.freq, self.rotary.magnitude) if self.rotary else (None, 1.0)
            n_.qkv_rotary_store(qq, c(k), c(v), self.k, self.v, pos, loc, freq, mag, self.H, self.G, self.D, self.Dv, 1e-6,
                                norm_values=False, qk_norm=2, q_norm_weight=qw.cuda(), k_norm_weight=kw.cuda())
            outs.append(n_.window_attention(qq, self.k, self.v, None, None, self.table, seq_params(2, self.held, n), self.H, self.G, self.D,
                                            self.Dv, self.size, 0, self.scale, self.matrix, keep_first=self.keep).float().cpu())
            self.held += n
        return torch.cat(outs)

    def oracle(self, q, k, v, qw, kw):
        T, r = q.shape[0], lambda t: t.to(self.dtype).double()
        qq = ko.rotate_halves(ko.rms(r(q).view(T, self.H, self.D), 1e-6) * qw.double(), self.rot)
        kk = ko.rotate_halves(ko.rms(r(k).view(T, self.G, self.D), 1e-6) * kw.double(), self.rot)
        vv = r(v).view(T, self.G, self.Dv)
        seen = ko.window_mask(T, {"size": self.size, "keep_first": self.keep} if self.size else None)
        out = torch.zeros(T, self.H, self.Dv, dtype=torch.float64)
        for h in range(self.H):
            g = h // (self.H // self.G)
            s = (qq[:, h] @ kk[:, g].T * self.scale).masked_fill(~seen, -math.inf)
            out[:, h] = torch.softmax(s, -1) @ vv[:, g]
        return out.reshape(T, -1)


def window_inputs(T, H, G, D, Dv, seed=3):
    g = torch.Generator().manual_seed(seed)
    return (*(torch.randn(T, n, generator=g) for n in (H * D, G * D, G * Dv)), 1 + 0.3 * torch.randn(D, generator=g),
            1 + 0.3 * torch.randn(D, generator=g))


@pytest.mark.parametrize("cut", CUTS)
@pytest.mark.parametrize("size,keep", [(5, 3), (64, 4), (1, 1), (16, 0), (33, 50), (400, 2), (0, 0)])
@pytest.mark.parametrize("shape", [(4, 2, 16, 24, 8), (3, 1, 24, 72, 10), (2, 2, 136, 200, 64)], ids=lambda s: "x".join(map(str, s)))
def test_window_with_kept_tokens_at_every_position(shape, size, keep, cut):
    """sharp scores (several units between keys) at every position of 150: one key more or less at the window's edge or among the
    kept tokens moves the output by far more than the bar"""
    H, G, D, Dv, dims = shape
    x = window_inputs(150, H, G, D, Dv)
    rot = {"dims": dims, "base": 100.0, "scaling": {"factor": 2.0, "low": 1.0, "high": 4.0, "original": 32}}
    b = WindowBench(H, G, D, Dv, size, keep, rot, scale=6.0 / D)
    want = b.oracle(*x)
    assert U.rel(b.run(*x, CUTS[cut]), want) < 2e-5
    if size in (5, 16):
        for other in ((size + 1, keep), (size - 1, keep), (size, keep + 1)):
            assert U.rel(WindowBench(H, G, D, Dv, *other, rot, scale=6.0 / D).oracle(*x), want) > 1e-2


@pytest.mark.parametrize("matrix", [False, True], ids=["vector", "matrix"])
def test_loud_keys_around_the_window_and_the_kept_tokens(matrix):
    """loud keys at position 3 (the last kept one), 4 (the first that is not) and 200 in a window of 70 among 500 tokens: each is
    heard exactly where it may be, at the edges and far from them, in prompts and decoded"""
    H, G, D, Dv, size, keep, T = 2, 1, 64, 64, 70, 4, 500
    q, k, v, qw, kw = window_inputs(T, H, G, D, Dv, seed=2)
    qw, kw = torch.ones(D), torch.ones(D)
    v *= 0.01
    q[:] = 0.1 * q
    k[:] = 0.1 * k
    q[:, 0] = q[:, 64] = 6.0
    k[:, 0] = 0.0
    marks = {3: 5, 4: 6, 200: 7}                                          # position -> its value's coordinate
    for p, col in marks.items():
        k[p] = 0.0
        k[p, 0], v[p] = 8.0, 0.0
        v[p, col] = 50.0
    heard = lambda out, p: {h: float(out[p, c]) > 5 for h, c in marks.items()}
    dtype = torch.bfloat16 if matrix else torch.float32
    for sizes in ([T], [250, 1], [64], [71, 2, 1], [2]):
        b = WindowBench(H, G, D, Dv, size, keep, dtype=dtype, matrix=matrix, scale=0.5)
        got = b.run(q, k, v, qw, kw, sizes)
        assert U.rel(got, b.oracle(q, k, v, qw, kw)) < (2e-5 if not matrix else 1.2e-2)
        for p, want in ((2, (0, 0, 0)), (3, (1, 0, 0)), (4, (1, 1, 0)), (73, (1, 1, 0)), (74, (1, 0, 0)), (199, (1, 0, 0)),
                        (200, (1, 0, 1)), (269, (1, 0, 1)), (270, (1, 0, 0)), (499, (1, 0, 0))):
            assert tuple(heard(got, p).values()) == tuple(map(bool, want)), (p, sizes)


@pytest.mark.parametrize("sizes", [[200], [17, 2, 64, 1, 1, 33, 16, 5], [3]], ids=["whole", "mixed", "threes"])
@pytest.mark.parametrize("size,keep", [(16, 3), (40, 0), (15, 17), (1, 1)])
@pytest.mark.parametrize("shape", [(8, 2, 128, 128), (4, 4, 64, 128), (6, 1, 128, 64)], ids=lambda s: "x".join(map(str, s)))
def test_matrix_core_windows_against_the_oracle(shape, size, keep, sizes):
    x = window_inputs(200, *shape, seed=7)
    b = WindowBench(*shape, size, keep, dtype=torch.bfloat16, scale=4.0 / shape[2])
    got = b.run(*x, sizes)
    assert torch.isfinite(got).all() and U.rel(got, b.oracle(*x)) < 1.5e-2


# ------------------------------------------------------------------------------------------------ the whole model
@pytest.fixture(scope="module")
def full(tmp_path_factory):
    cfg = U.full_config()
    folder, w = U.make_model(tmp_path_factory.mktemp("full"), cfg, seed=11)
    toks = U.tokens(130, cfg["vocab"], 12)
    lay = []
    want = ko.forward(toks, w, cfg, lay)
    return cfg, folder, w, toks, want, lay


def test_whole_prompt_with_the_stream_after_every_layer(full):
    cfg, folder, w, toks, want, lay = full
    eng = engine(folder)
    eng.runner.model.capture_layers = []
    got = run_whole(eng, toks)
    for i, (a, b) in enumerate(zip(eng.runner.model.capture_layers, lay)):
        assert U.rel(a, b) < F32_BAR, i
    assert U.rel(got, want) < F32_BAR
    eng.runner.model.capture_layers = None
    assert U.rel(run_whole(eng, toks, "again"), want) < F32_BAR            # on rows and slots used before


@pytest.mark.parametrize("sizes", [[130], [1], [5, 2, 1, 1, 40, 3, 1]], ids=["whole", "decode", "mixed"])
def test_serving_precision(full, sizes):
    cfg, folder, w, toks, want, _ = full
    got = run_portions(engine(folder, dtype=torch.bfloat16), toks, sizes)
    err = (got.double().cpu() - want).abs().amax(-1) / want.abs().max()
    assert float(err.median()) < 3e-2 and float(err.max()) < 0.12


@pytest.mark.parametrize("graphs", [False, True], ids=["eager", "graphs"])
def test_decoding_from_the_first_token(full, graphs):
    """130 single-token steps: the first is a first token on a fresh slot, every later one a decode step through the caches,
    convolution states and matrix states"""
    cfg, folder, w, toks, want, _ = full
    assert U.rel(run_portions(engine(folder, graphs=graphs), toks, [1]), want) < F32_BAR


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["fp32", "bf16"])
def test_long_decoding_behind_a_prompt(tmp_path, dtype):
    """360 decoded tokens: the window of 48 passes over prompt and decoded tokens alike, latent rows cross many key tiles"""
    cfg = U.config([(U.latent(4, 16, 8, 24, 40), U.dense(40)), (U.parallel(2, 1, 64, 64, 2, 1, 16, 24, size=48, keep=4), None),
                    (U.latent(2, 24, 8, 16, 40, kv_from=0), U.dense(24))], width=64, vocab=61)
    folder, w = U.make_model(tmp_path, cfg, seed=8)
    toks = U.tokens(400, 61, 9)
    want = ko.forward(toks, w, cfg)
    got = run_portions(engine(folder, dtype=dtype, graphs=True), toks, [40, 1])
    if dtype == torch.float32:
        assert U.rel(got, want) < F32_BAR
    else:
        err = (got.double().cpu() - want).abs().amax(-1) / want.abs().max()
        assert float(err.median()) < 3e-2 and float(err.max()) < 0.12


@pytest.mark.parametrize("sizes", [[2], [3, 2, 17, 1, 1, 64, 5, 1], [64, 2, 1], [15, 16, 17, 1], [10, 1, 1, 12, 23, 1]],
                         ids=["pairs", "mixed", "big-then-small", "near-16", "near-the-windows"])
def test_portions_of_prompts(full, sizes):
    cfg, folder, w, toks, want, _ = full
    assert U.rel(run_portions(engine(folder), toks, sizes), want) < F32_BAR


def test_garbage_in_reused_rows_and_slots_is_never_read(full):
    cfg, folder, w, toks, want, _ = full
    for dtype in (torch.float32, torch.bfloat16):
        eng = engine(folder, dtype=dtype)
        for spec in eng.runner.state_pool.named.values():
            for t in spec.values():
                t.fill_(float("nan"))
        for b in eng.runner.token_to_kv_pool._all():
            b.fill_(float("nan"))
        assert U.rel(run_portions(eng, toks[:60], [7, 1]), want[:60]) < (F32_BAR if dtype == torch.float32 else 0.12)


@pytest.mark.parametrize("graphs", [False, True], ids=["eager", "graphs"])
def test_unequal_batches_with_rows_and_slots_reused(full, graphs):
    """seven requests of unequal length through three rows and a pool that holds far fewer tokens than their sum: portions
    of some beside single tokens of others, pauses, rows and slots handed on; every request's logits must be what it gets
    alone"""
    cfg, folder, w, _, _, _ = full
    reqs = {f"r{i}": U.tokens(n, cfg["vocab"], 20 + i) for i, n in enumerate([45, 3, 70, 1, 26, 58, 12])}
    want = {r: ko.forward(t, w, cfg) for r, t in reqs.items()}
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
            n = plan[r].pop(0) if plan[r] else 1
            n = min(n, len(reqs[r]) - fed[r])
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
    reqs = {f"q{i}": U.tokens(3 + i % 19, cfg["vocab"], 300 + i) + U.tokens(6, cfg["vocab"], 900 + i) for i in range(40)}
    engs = [engine(folder, dtype=dtype, tokens=1100, slots=40, graphs=g) for g in (True, False)]
    for eng in engs:
        eng.step([entry(r, t[:-6], []) for r, t in reqs.items()])                     # the prompts, one extend batch
    outs = [[], []]
    for k in range(6):
        for eng, out in zip(engs, outs):
            out.append(eng.step([entry(r, [t[len(t) - 6 + k]]) for r, t in reqs.items()], list(reqs) if k == 5 else []))
            torch.cuda.synchronize()
    bar = 1e-5 if dtype == torch.float32 else 3e-2
    for k in range(6):
        assert U.rel(outs[0][k], outs[1][k]) < bar, k
    if dtype == torch.float32:
        want = torch.stack([ko.forward(t, w, cfg)[-6:] for t in reqs.values()], 1)    # [step, request, vocab]
        assert U.rel(torch.stack(outs[0]), want) < F32_BAR


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
            lg = ko.forward(p + ref[:agree], w, cfg)[-1]
            assert float(lg[ref[agree]] - lg[out[agree]]) < 1e-3 * float(lg.abs().max()), (agree, out, ref)
        else:
            assert out == ref
    sampled = eng.generate(prompts[:2], SamplingParams(max_new_tokens=6, temperature=0.8, top_p=0.9, top_k=20))
    assert all(len(o) == 6 and all(0 <= t < cfg["vocab"] for t in o) for o in sampled)


def test_the_learned_positions_bound_a_request(tmp_path):
    cfg = U.config([(U.latent(2, 8, 4, 8, 16), None)], width=48, vocab=61, positions=40)
    folder, w = U.make_model(tmp_path, cfg, seed=1)
    eng = engine(folder, tokens=200)
    toks = U.tokens(41, 61, 2)
    assert U.rel(eng.step([entry("a", toks[:40])]), ko.forward(toks[:40], w, cfg)) < F32_BAR       # the last row of the table
    with pytest.raises(ValueError, match="context"):
        eng.step([entry("a", toks[40:])])
    with pytest.raises(ValueError, match="context"):
        eng.generate([toks[:30]], max_new_tokens=12)
    eng.step([], ["a"])
    assert len(eng.generate([toks[:30]], max_new_tokens=11)[0]) == 11                             # the last one is not fed


@pytest.mark.parametrize("seed", range(12))
def test_designs_drawn_at_random(tmp_path, seed):
    """layer order, shared rows, sizes and constants drawn at random: whole prompt, then portions of random sizes with single
    tokens between them, both against the oracle; the same portions in bf16"""
    import random
    cfg = U.random_config(100 + seed)
    folder, w = U.make_model(tmp_path, cfg, seed=seed)
    toks = U.tokens(90, cfg["vocab"], seed)
    want = ko.forward(toks, w, cfg)
    assert U.rel(run_whole(engine(folder), toks), want) < F32_BAR, cfg
    r = random.Random(seed)
    sizes = [r.choice([1, 1, 2, 3, 7, 16, 29]) for _ in range(40)]
    assert U.rel(run_portions(engine(folder), toks, sizes), want) < F32_BAR, (sizes, cfg)
    got = run_portions(engine(folder, dtype=torch.bfloat16), toks, sizes)
    err = (got.double().cpu() - want).abs().amax(-1) / want.abs().max()
    assert float(err.median()) < (4e-2 if cfg["postln_alpha"] > 1 else 0.1), (sizes, cfg)      # (alpha 1: a layer doubles the noise)


def test_sizes_that_are_one_or_equal(tmp_path):
    """a model whose sizes are 1 or equal where the others' differ: one head everywhere, key width = value width = latent rank =
    model width, rotation over the whole head, alpha 1, one tap, as many kept tokens as the window holds"""
    cfg = U.config([
        (U.latent(1, 16, 16, 16, 16, scale=1.0), U.dense(16)),
        (U.parallel(1, 1, 16, 16, 1, 1, 16, 16, size=4, keep=4, dims=16, conv=1, scale=1.0), U.dense(16)),
        (U.latent(1, 16, 16, 16, 16, scale=1.0, kv_from=0), None),
        (U.parallel(1, 1, 16, 16, 1, 1, 16, 16, size=1, keep=0, dims=16, conv=1, scale=1.0), None),
    ], width=16, vocab=17, alpha=1.0, positions=64)
    folder, w = U.make_model(tmp_path, cfg, seed=4)
    toks = U.tokens(50, 17, 3)
    want = ko.forward(toks, w, cfg)
    assert U.rel(run_whole(engine(folder), toks), want) < F32_BAR
    assert U.rel(run_portions(engine(folder), toks, [3, 1]), want) < F32_BAR
