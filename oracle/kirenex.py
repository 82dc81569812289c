"""CPU oracle of the Kirenex design: one plain, slow function per mechanism, written from the design's equations.

TEST INFRASTRUCTURE ONLY: nothing under scratchpad_amd/ imports this, and this imports nothing from there.  Every
function works on ONE whole sequence in float64 (or the dtype it is given) and keeps no cache and no state: a sequence
is recomputed from its first token, which is what makes it a reference for caches, states, portions and batches.

Notation: T tokens, W model width, x the residual stream [T, W], N(z) = z / rms(z).  A layer is
    x <- N(a x + mixer(x)) w1;    x <- N(a x + ff(x)) w2
with a one constant of the model.  The mixer is, layer by layer, attention over a shared latent of the keys and values
(its own, or the one another layer made), or two mixers on the same input, each normed over the width and averaged: softmax
attention that sees a window and the first tokens, and a delta rule with one decay per head.
"""
import math
from typing import Dict, List, Optional

import torch


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.where(z > 30, z, torch.log1p(torch.exp(torch.clamp(z, max=30))))


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


# ----------------------------------------------------------------------------------------------- embedding
def embed(tokens: List[int], w: Dict[str, torch.Tensor]) -> torch.Tensor:
    """token rows plus the learned row of the position"""
    return w["embed"][torch.tensor(tokens)] + w["pos"][:len(tokens)]


# ----------------------------------------------------------------------------------------------- rotary
def rotary_frequencies(rot: dict) -> torch.Tensor:
    """one per pair: base^(-2i/dims), bent by wavelength where ``scaling`` = {factor, low, high, original} is given"""
    dims, base = int(rot["dims"]), float(rot["base"])
    out, sc = [], rot.get("scaling")
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if sc:
            factor, low, high, orig = (float(sc[k]) for k in ("factor", "low", "high", "original"))
            turns = orig * f / (2 * math.pi)                       # full turns inside the original context
            if turns < low:
                f = f / factor
            elif turns <= high:
                s = (turns - low) / (high - low)
                f = (1 - s) * f / factor + s * f
        out.append(f)
    return torch.tensor(out, dtype=torch.float64)


def angles(T: int, rot: dict, dtype):
    a = torch.arange(T, dtype=torch.float64)[:, None] * rotary_frequencies(rot)[None, :]
    return torch.cos(a).to(dtype)[:, None, :], torch.sin(a).to(dtype)[:, None, :]


def rotate_halves(x: torch.Tensor, rot: Optional[dict]) -> torch.Tensor:
    """x [T, heads, n], row t at position t: coordinate i < dims / 2 turns with coordinate i + dims / 2; the rest pass"""
    if not rot or int(rot["dims"]) == 0:
        return x
    dims = int(rot["dims"])
    c, s = angles(x.shape[0], rot, x.dtype)
    u, v = x[..., :dims // 2], x[..., dims // 2:dims]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., dims:]], -1)


def rotate_neighbours(x: torch.Tensor, rot: Optional[dict]) -> torch.Tensor:
    """x [T, heads, n]: coordinate 2i turns with coordinate 2i + 1, i < dims / 2; the rest pass"""
    if not rot or int(rot["dims"]) == 0:
        return x
    dims = int(rot["dims"])
    c, s = angles(x.shape[0], rot, x.dtype)
    out = x.clone()
    out[..., 0:dims:2] = x[..., 0:dims:2] * c - x[..., 1:dims:2] * s
    out[..., 1:dims:2] = x[..., 1:dims:2] * c + x[..., 0:dims:2] * s
    return out


# ----------------------------------------------------------------------------------------------- latent attention
def latent(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float):
    """what a layer keeps of a token: (normed latent [T, rank], rotated key part [T, rot_dim])"""
    C = int(m["kv_rank"])
    a = h @ w[f"{p}.dkv"].T
    return rms(a[:, :C], eps) * w[f"{p}.dkv.norm"], rotate_neighbours(a[:, None, C:], m["rot"])[:, 0]


def latent_attention(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict, kept) -> torch.Tensor:
    """kept: the pair ``latent`` made, of this layer or of the layer it takes it from"""
    T = h.shape[0]
    H, D, R, Dv = (int(m[k]) for k in ("heads", "dim", "rot_dim", "vdim"))
    c, kr = kept
    q = (h @ w[f"{p}.q"].T).reshape(T, H, D + R)
    qu, qr = q[..., :D], rotate_neighbours(q[..., D:], m["rot"])
    ku, v = (c @ w[f"{p}.uk"].T).reshape(T, H, D), (c @ w[f"{p}.uv"].T).reshape(T, H, Dv)
    seen = torch.ones(T, T, dtype=torch.bool).tril()
    out = torch.zeros(T, H, Dv, dtype=h.dtype)
    for n in range(H):
        s = (qu[:, n] @ ku[:, n].T + qr[:, n] @ kr.T) * float(m["scale"])
        out[:, n] = torch.softmax(s.masked_fill(~seen, -math.inf), -1) @ v[:, n]
    return (out.reshape(T, H * Dv) * torch.sigmoid(h @ w[f"{p}.g"].T)) @ w[f"{p}.o"].T


# ----------------------------------------------------------------------------------------------- window + first tokens
def window_mask(T: int, mask: Optional[dict]) -> torch.Tensor:
    """[T, T] bool: query i sees key j"""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    if not mask:
        return j <= i
    return (j <= i) & ((i - j < int(mask["size"])) | (j < int(mask.get("keep_first", 0))))


def window_attention(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, G, D, Dv = (int(m[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
    q = rotate_halves(rms((h @ w[f"{p}.q"].T).reshape(T, H, D), eps) * w[f"{p}.q.norm"], m.get("rot"))
    k = rotate_halves(rms((h @ w[f"{p}.k"].T).reshape(T, G, D), eps) * w[f"{p}.k.norm"], m.get("rot"))
    v = (h @ w[f"{p}.v"].T).reshape(T, G, Dv)
    seen = window_mask(T, m.get("mask"))
    out = torch.zeros(T, H, Dv, dtype=h.dtype)
    for n in range(H):
        g = n // (H // G)
        s = (q[:, n] @ k[:, g].T) * float(m["scale"])
        out[:, n] = torch.softmax(s.masked_fill(~seen, -math.inf), -1) @ v[:, g]
    return out.reshape(T, H * Dv) @ w[f"{p}.o"].T


# ----------------------------------------------------------------------------------------------- gated delta rule
def causal_conv(u: torch.Tensor, taps: torch.Tensor) -> torch.Tensor:
    """u [T, n], taps [n, K]: out[t] = sum_j taps[:, j] u[t - (K - 1) + j], zeros before the start"""
    T, K = u.shape[0], taps.shape[1]
    pad = torch.cat([torch.zeros(K - 1, u.shape[1], dtype=u.dtype), u], 0)
    return sum(pad[j:j + T] * taps[:, j] for j in range(K))


def unit(x: torch.Tensor) -> torch.Tensor:
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_scan(q, k, v, beta, decay) -> torch.Tensor:
    """one head: unit q (scaled) and k [T, D], v [T, Dv], beta and decay [T] -> o [T, Dv]"""
    S = torch.zeros(k.shape[1], v.shape[1], dtype=v.dtype)
    out = torch.zeros_like(v)
    for t in range(v.shape[0]):
        S = decay[t] * S
        S = S + torch.outer(k[t], beta[t] * (v[t] - S.T @ k[t]))
        out[t] = S.T @ q[t]
    return out


def delta_rule(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, G, D, Dv = (int(m[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
    conv = lambda n: silu(causal_conv(h @ w[f"{p}.{n}"].T, w[f"{p}.{n}.conv"]))
    q = unit(conv("q").reshape(T, G, D)) * D ** -0.5
    k = unit(conv("k").reshape(T, G, D))
    v = conv("v").reshape(T, H, Dv)
    beta = torch.sigmoid(h @ w[f"{p}.b"].T)
    decay = torch.exp(-torch.exp(w[f"{p}.A_log"]) * softplus(h @ w[f"{p}.a"].T + w[f"{p}.dt_bias"]))
    o = torch.stack([delta_scan(q[:, n // (H // G)], k[:, n // (H // G)], v[:, n], beta[:, n], decay[:, n]) for n in range(H)], 1)
    gate = silu(h @ w[f"{p}.g"].T).reshape(T, H, Dv)
    return (rms(o, eps) * w[f"{p}.norm"] * gate).reshape(T, H * Dv) @ w[f"{p}.o"].T


def average_of_normed(a, b, wa, wb, eps: float) -> torch.Tensor:
    return 0.5 * (rms(a, eps) * wa + rms(b, eps) * wb)


def parallel(h, w, p: str, m: dict, eps: float) -> torch.Tensor:
    return average_of_normed(window_attention(h, w, f"{p}.left", m["left"], eps), delta_rule(h, w, f"{p}.right", m["right"], eps),
                             w[f"{p}.left.out"], w[f"{p}.right.out"], eps)


# ----------------------------------------------------------------------------------------------- model
def feed_forward(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str) -> torch.Tensor:
    return (gelu_tanh(h @ w[f"{p}.gate"].T) * (h @ w[f"{p}.up"].T)) @ w[f"{p}.down"].T


def post_norm(x, y, weight, alpha: float, eps: float) -> torch.Tensor:
    return rms(alpha * x + y, eps) * weight


def forward(tokens: List[int], w: Dict[str, torch.Tensor], cfg: dict, capture: Optional[list] = None,
            last_only: bool = False) -> torch.Tensor:
    """logits [T, vocab] of one sequence ([1, vocab] with ``last_only``); ``capture`` collects the stream after every layer"""
    eps, alpha = float(cfg["norm"]["eps"]), float(cfg["postln_alpha"])
    x = embed(tokens, w)
    kept = {}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}", layer["mixer"]
        if layer["type"] == "latent_attention":
            j = m.get("kv_from")
            if j is None:
                kept[i] = latent(x, w, f"{p}.mix", m, eps)
                j = i
            y = latent_attention(x, w, f"{p}.mix", m, kept[int(j)])
        else:
            y = parallel(x, w, f"{p}.mix", m, eps)
        x = post_norm(x, y, w[f"{p}.norm1"], alpha, eps)
        if layer.get("mlp"):
            x = post_norm(x, feed_forward(x, w, f"{p}.mlp"), w[f"{p}.norm2"], alpha, eps)
        if capture is not None:
            capture.append(x.clone())
    if last_only:
        x = x[-1:]
    return rms(x, eps) * w["final.norm"] @ w["head"].T


# ----------------------------------------------------------------------------------------------- random weights
def tensor_shapes(cfg: dict) -> Dict[str, tuple]:
    W, V = int(cfg["width"]), int(cfg["vocab"])
    out = {"embed": (V, W), "pos": (int(cfg["max_positions"]), W), "head": (V, W), "final.norm": (W,)}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}", layer["mixer"]
        out[f"{p}.norm1"] = (W,)
        if layer["type"] == "latent_attention":
            H, D, R, Dv, C = (int(m[k]) for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
            out.update({f"{p}.mix.q": (H * (D + R), W), f"{p}.mix.uk": (H * D, C), f"{p}.mix.uv": (H * Dv, C),
                        f"{p}.mix.g": (H * Dv, W), f"{p}.mix.o": (W, H * Dv)})
            if m.get("kv_from") is None:
                out.update({f"{p}.mix.dkv": (C + R, W), f"{p}.mix.dkv.norm": (C,)})
        else:
            a, b = m["left"], m["right"]
            H, G, D, Dv = (int(a[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
            L = f"{p}.mix.left"
            out.update({f"{L}.q": (H * D, W), f"{L}.k": (G * D, W), f"{L}.v": (G * Dv, W), f"{L}.q.norm": (D,),
                        f"{L}.k.norm": (D,), f"{L}.o": (W, H * Dv), f"{L}.out": (W,)})
            H, G, D, Dv, K = (int(b[k]) for k in ("heads", "kv_heads", "dim", "vdim", "conv"))
            R = f"{p}.mix.right"
            for n, rows in (("q", G * D), ("k", G * D), ("v", H * Dv)):
                out.update({f"{R}.{n}": (rows, W), f"{R}.{n}.conv": (rows, K)})
            out.update({f"{R}.b": (H, W), f"{R}.a": (H, W), f"{R}.A_log": (H,), f"{R}.dt_bias": (H,), f"{R}.norm": (Dv,),
                        f"{R}.g": (H * Dv, W), f"{R}.o": (W, H * Dv), f"{R}.out": (W,)})
        if layer.get("mlp"):
            ff = int(layer["mlp"]["ff"])
            out.update({f"{p}.norm2": (W,), f"{p}.mlp.gate": (ff, W), f"{p}.mlp.up": (ff, W), f"{p}.mlp.down": (W, ff)})
    return out


def random_weights(cfg: dict, seed: int, dtype=torch.float64) -> Dict[str, torch.Tensor]:
    """weights of a scale at which every mechanism reaches the logits, already rounded to bfloat16 (checkpoints hold that)"""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        z = torch.randn(*shape, generator=g, dtype=torch.float64)
        leaf = name.rsplit(".", 1)[-1]
        if leaf in ("norm", "norm1", "norm2", "out"):
            z = 1.0 + 0.3 * z
        elif leaf == "conv":
            z = 0.6 * z
        elif leaf == "A_log":
            z = 0.7 * z - 1.5
        elif leaf == "dt_bias":
            z = z - 1.0
        elif leaf == "pos":
            z = 0.7 * z
        elif leaf != "embed":
            z = 1.3 * z / math.sqrt(shape[-1])
        out[name] = z.to(torch.bfloat16).to(dtype)
    return out
