"""The Kirenex kernels at the layer sizes of real models (bf16 and fp32), each against a plain fp32 torch expression of the
same operation evaluated on the GPU (products of a head taken one by one, in fp32): several requests of unequal length in one
launch, a second launch that goes on from what the first one left.  Every case prints its name before it launches."""
import pytest
import torch

from tests.test_gpu_toredra_kernels import DEV, announce, close, rms, seq_extend

pytestmark = pytest.mark.gpu


@pytest.mark.parametrize("dtype,bar", [(torch.float32, 1e-4), (torch.bfloat16, 2e-2)])
@pytest.mark.parametrize("H,G,D,Dv", [(16, 8, 128, 128), (8, 8, 64, 256), (32, 4, 64, 64), (4, 2, 256, 128)])
def test_head_delta_scan_at_model_size(dtype, bar, H, G, D, Dv):
    from scratchpad_amd import _native
    lens, slots = [500, 1, 223], [3, 1, 4]
    T, rep = sum(lens), H // G
    announce("head_delta_scan", dtype, "heads", H, "kv heads", G, "dim", D, "vdim", Dv, "tokens", lens)
    g = torch.Generator(device=DEV).manual_seed(0)
    rn = lambda *s: torch.randn(*s, generator=g, device=DEV)
    state = torch.full((6, H, D, Dv), float("nan"), device=DEV)
    S = {s: torch.zeros(H, D, Dv, device=DEV) for s in slots}
    A, dt, nw = rn(H) * 0.5 - 2, rn(H), torch.rand(Dv, generator=g, device=DEV) + 0.5
    for launch, prefixes in enumerate(([0, 0, 0], lens)):                      # the second launch goes on from the first's states
        q, k = (rn(T, G * D).to(dtype) for _ in range(2))
        v, gate = (rn(T, H * Dv).to(dtype) for _ in range(2))
        pre = rn(T, 2 * H)
        got = _native.head_delta_scan(q, k, v, gate, pre, dt, A, nw, state, seq_extend(lens, prefixes, slots), H, G, D, Dv, 1e-5)
        want = torch.empty(T, H, Dv, device=DEV)
        unit = lambda x: x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)
        at = 0
        for m, slot in zip(lens, slots):
            qq, kk = (unit(t[at:at + m].float().view(m, G, D)).repeat_interleave(rep, 1) for t in (q, k))
            vv, bb = v[at:at + m].float().view(m, H, Dv), torch.sigmoid(pre[at:at + m, :H])
            ww = torch.exp(-torch.exp(A) * torch.nn.functional.softplus(pre[at:at + m, H:] + dt))
            for t in range(m):
                Sd = ww[t].view(H, 1, 1) * S[slot]
                u = bb[t].unsqueeze(-1) * (vv[t] - (Sd * kk[t].unsqueeze(-1)).sum(1))
                S[slot] = Sd + kk[t].unsqueeze(-1) * u.unsqueeze(-2)
                want[at + t] = (S[slot] * qq[t].unsqueeze(-1)).sum(1) * D ** -0.5
            close(state[slot], S[slot], 1e-3 if dtype == torch.float32 else bar)
            at += m
        close(got, (rms(want, 1e-5) * nw).reshape(T, H * Dv) * torch.nn.functional.silu(gate.float()), bar)
    assert torch.isnan(state[0]).all() and torch.isnan(state[2]).all()          # no other slot was touched


def rotate_pairs(x, pos, freq):
    """interleaved pairs of x [T, heads, R] in fp32"""
    ang = pos.float()[:, None] * freq
    c, s = ang.cos()[:, None], ang.sin()[:, None]
    u, v = x[..., 0::2], x[..., 1::2]
    return torch.stack([u * c - v * s, v * c + u * s], -1).flatten(-2)


@pytest.mark.parametrize("dtype,bar", [(torch.float32, 1e-4), (torch.bfloat16, 2e-2)])
@pytest.mark.parametrize("H,D,R,Dv,C", [(16, 128, 64, 128, 512), (32, 64, 32, 64, 256), (8, 96, 32, 80, 128), (64, 128, 64, 128, 512)])
def test_latent_attention_at_model_size(dtype, bar, H, D, R, Dv, C):
    """store, folded query product, attention, value product with the output gate, as the model runs them: one launch of portions,
    then single tokens; against keys and values formed head by head"""
    from scratchpad_amd import _native
    from scratchpad_amd.layers import AngleRotary
    lens, slots = [400, 1, 223], [3, 1, 4]
    announce("latent attention", dtype, "heads", H, "dim", D, R, "vdim", Dv, "rank", C, "tokens", lens)
    g = torch.Generator(device=DEV).manual_seed(0)
    rn = lambda *s: torch.randn(*s, generator=g, device=DEV)
    rot = AngleRotary(R, 10000.0).to(DEV)
    uk, uv = (rn(H, D, C) * C ** -0.5).to(dtype), (rn(H, Dv, C) * C ** -0.5).to(dtype)
    uk_t, nw, scale = uk.transpose(1, 2).contiguous(), 1 + 0.3 * rn(C), (D + R) ** -0.5
    P, width = 800, 500
    pool = torch.full((P + 1, C + R), float("nan"), dtype=dtype, device=DEV)
    free = torch.randperm(P, generator=g, device=DEV) + 1
    table = torch.zeros(6, width, dtype=torch.int32, device=DEV)
    cs, krs, used = {s: [] for s in slots}, {s: [] for s in slots}, 0
    for prefixes, new in (([0, 0, 0], lens), (lens, [1, 1, 1]), ([n + 1 for n in lens], [1, 1, 1])):
        T = sum(new)
        a = rn(T, H * (D + R) + C + R + H * Dv).to(dtype)
        pos = torch.cat([torch.arange(p, p + n, device=DEV) for p, n in zip(prefixes, new)])
        loc = free[used:used + T]
        used += T
        at = 0
        for p, n, slot in zip(prefixes, new, slots):
            table[slot, p:p + n] = loc[at:at + n].to(torch.int32)
            at += n
        nq = H * (D + R)
        q = a[:, :nq].view(T, H, D + R)
        q0 = q.float().clone()
        seq = seq_extend(new, prefixes, slots) if T > 3 else _native.SeqParams(
            torch.tensor(slots, device=DEV), torch.tensor([p + 1 for p in prefixes], device=DEV))
        _native.latent_kv_store(pool, a[:, nq:nq + C + R], nw, pos, rot.freq, 1.0, loc, C, 1e-5, q=q, q_offset=D)
        q_lat = _native.head_linear(q[:, :, :D], uk_t)
        o_lat = _native.latent_attention(q_lat, q[:, :, D:], pool, table, seq, scale, token_major=True)
        got = _native.head_linear(o_lat, uv, gate=a[:, nq + C + R:])
        dkv = a[:, nq:nq + C + R].float()
        c_new, kr_new = rms(dkv[:, :C], 1e-5) * nw, rotate_pairs(dkv[:, None, C:], pos, rot.freq)[:, 0]
        qr = rotate_pairs(q0[..., D:], pos, rot.freq)
        want, at = torch.empty(T, H, Dv, device=DEV), 0
        for p, n, slot in zip(prefixes, new, slots):
            cs[slot].append(c_new[at:at + n])
            krs[slot].append(kr_new[at:at + n])
            c, kr = torch.cat(cs[slot]), torch.cat(krs[slot])
            hide = torch.arange(c.shape[0], device=DEV)[None] > torch.arange(p, p + n, device=DEV)[:, None]
            for h in range(H):
                s = (q0[at:at + n, h, :D] @ (c @ uk[h].float().T).T + qr[at:at + n, h] @ kr.T) * scale
                want[at:at + n, h] = torch.softmax(s.masked_fill(hide, float("-inf")), -1) @ (c @ uv[h].float().T)
            at += n
        want = want.reshape(T, H * Dv) * torch.sigmoid(a[:, nq + C + R:].float())
        close(got.reshape(T, H * Dv), want, bar)


@pytest.mark.parametrize("dtype,bar", [(torch.float32, 1e-4), (torch.bfloat16, 2e-2)])
@pytest.mark.parametrize("H,G,D,dims,size,keep", [(16, 4, 128, 64, 128, 4), (32, 8, 64, 64, 1, 3), (8, 8, 128, 32, 300, 0)])
def test_window_with_kept_tokens_at_model_size(dtype, bar, H, G, D, dims, size, keep):
    from scratchpad_amd import _native
    from scratchpad_amd.layers import HalfAngleRotary
    lens, slots = [700, 1, 323], [3, 1, 4]
    T = sum(lens)
    announce("window", dtype, "heads", H, "kv heads", G, "dim", D, "window", size, "kept", keep, "tokens", lens)
    g = torch.Generator(device=DEV).manual_seed(0)
    rn = lambda *s: torch.randn(*s, generator=g, device=DEV)
    a, qn, kn = rn(T, (H + 2 * G) * D).to(dtype), 1 + 0.3 * rn(D), 1 + 0.3 * rn(D)
    rot = HalfAngleRotary(dims, 10000.0, {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 256}).to(DEV)
    pos = torch.cat([torch.arange(m, device=DEV) for m in lens])
    loc = torch.randperm(T, generator=g, device=DEV) + 1
    table = torch.zeros(6, 800, dtype=torch.int32, device=DEV)
    kpool, vpool = (torch.full((T + 1, G * D), float("nan"), dtype=dtype, device=DEV) for _ in range(2))
    want, at, half = torch.empty(T, H, D, device=DEV), 0, dims // 2

    def make(z, nw):                                           # [m, heads, D] -> normed, rotated
        z = rms(z, 1e-5) * nw
        ang = torch.arange(z.shape[0], device=DEV).float()[:, None] * rot.freq
        c, s = ang.cos()[:, None], ang.sin()[:, None]
        u, v = z[..., :half], z[..., half:dims]
        return torch.cat([u * c - v * s, v * c + u * s, z[..., dims:]], -1)
    for m, slot in zip(lens, slots):
        table[slot, :m] = loc[at:at + m].to(torch.int32)
        q, k, v = (t.float().view(m, -1, D) for t in (a[at:at + m, :H * D], a[at:at + m, H * D:(H + G) * D], a[at:at + m, (H + G) * D:]))
        q, k = make(q, qn), make(k, kn)
        i, j = torch.arange(m, device=DEV)[:, None], torch.arange(m, device=DEV)[None]
        seen = (j <= i) & ((i - j < size) | (j < keep))
        for h in range(H):
            s = (q[:, h] @ k[:, h // (H // G)].T * 0.2).masked_fill(~seen, float("-inf"))
            want[at:at + m, h] = torch.softmax(s, -1) @ v[:, h // (H // G)]
        at += m
    q = a[:, :H * D]
    _native.qkv_rotary_store(q, a[:, H * D:(H + G) * D], a[:, (H + G) * D:], kpool, vpool, pos, loc, rot.freq, 1.0, H, G, D, D, 1e-5,
                             norm_values=False, qk_norm=2, q_norm_weight=qn, k_norm_weight=kn)
    got = _native.window_attention(q, kpool, vpool, None, None, table, seq_extend(lens, [0, 0, 0], slots), H, G, D, D, size, 0, 0.2,
                                   keep_first=keep)
    close(got, want.reshape(T, H * D), bar)


@pytest.mark.parametrize("dtype,bar", [(torch.float32, 2e-5), (torch.bfloat16, 1e-2)])
@pytest.mark.parametrize("T", [8, 4096])
def test_join_activation_and_convolution_at_model_size(dtype, bar, T):
    from scratchpad_amd import _native
    W, C, K = 4096, 8192, 4
    announce("post_norm of two branches / gelu_tanh_and_mul / causal_conv_silu", dtype, "rows", T)
    g = torch.Generator(device=DEV).manual_seed(1)
    rn = lambda *s: torch.randn(*s, generator=g, device=DEV)
    x, prod = rn(T, W), rn(T, 2 * W).to(dtype)
    a, b = prod[:, :W], prod[:, W:]                                            # views of one product
    wa, wb, w = (rn(W) * 0.2 + 1 for _ in range(3))
    want = rms(2.5 * x + 0.5 * (rms(a.float(), 1e-5) * wa + rms(b.float(), 1e-5) * wb), 1e-5) * w
    xs = x.clone()
    lo = _native.post_norm(xs, a, w, 1e-5, 2.5, dtype, b=b, wa=wa, wb=wb)
    close(xs, want, 2e-5)
    close(lo, want, bar)
    close(_native.gelu_tanh_and_mul(prod), torch.nn.functional.gelu(a.float(), approximate="tanh") * b.float(), bar)
    lens = [T] if T == 8 else [1500, 1, 2595]
    u, taps, state = rn(T, C).to(dtype), rn(C, K), torch.full((6, K - 1, C), float("nan"), device=DEV)
    got = _native.causal_conv_silu(u, taps, None, state, seq_extend(lens, [0] * len(lens), [3, 1, 4][:len(lens)]))
    at = 0
    for m, slot in zip(lens, [3, 1, 4]):
        pad = torch.cat([torch.zeros(K - 1, C, device=DEV), u[at:at + m].float()])
        close(got[at:at + m], torch.nn.functional.silu(sum(pad[j:j + m] * taps[:, j] for j in range(K))), bar)
        assert torch.equal(state[slot], pad[m:])
        at += m
