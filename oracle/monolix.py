"""CPU oracle of the Monolix design: one plain, slow function per mechanism, written from the design's equations.

TEST INFRASTRUCTURE ONLY: nothing under scratchpad_amd/ imports this, and this imports nothing from there.  Every
function works on ONE whole sequence in float64 (or the dtype it is given) and keeps no cache: a sequence is recomputed
from its first token, which is what makes it a reference for caches, portions and batches.

Notation: T tokens, W model width, x the residual stream [T, W], N(z, w) = z / rms(z) * (1 + w).  A layer is
    x <- N(a x + s1 * mixer(x), w1);    x <- N(a x + s2 * ff(x), w2)
with a one constant of the model and s1, s2 learned vectors.  The mixer is grouped-query softmax attention whose values
are its keys as projected; the feed-forward is a mixture of relu-square experts, some of which hand their input on, beside
a shared expert behind a scalar gate.
"""
import math
from typing import Dict, List, Optional

import torch


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def shifted_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """the stored weight is the distance of the gain from one"""
    return rms(x, eps) * (1 + w)


# ----------------------------------------------------------------------------------------------- rotary
def rotary_frequencies(rot: dict) -> torch.Tensor:
    dims, base = int(rot["dims"]), float(rot["base"])
    return torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=torch.float64)


def rotate(x: torch.Tensor, rot: Optional[dict]) -> torch.Tensor:
    """x [T, heads, D], row t at position t: coordinate i < dims / 2 turns with coordinate i + dims / 2; the rest pass"""
    if not rot or int(rot["dims"]) == 0:
        return x
    f = rotary_frequencies(rot).to(x.dtype)
    half = f.numel()
    ang = torch.arange(x.shape[0], dtype=x.dtype)[:, None] * f[None, :]
    c, s = torch.cos(ang)[:, None, :], torch.sin(ang)[:, None, :]
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * half:]], -1)


# ----------------------------------------------------------------------------------------------- attention
def attention(x: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float) -> torch.Tensor:
    T = x.shape[0]
    H, G, D, Dv = (int(m[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
    assert D == Dv, "values are keys"
    q = (x @ w[f"{p}.q"].T + w[f"{p}.q.b"]).reshape(T, H, D)
    k = (x @ w[f"{p}.k"].T + w[f"{p}.k.b"]).reshape(T, G, D)
    v = k                                                          # before the norm and the rotation
    q = rotate(rms(q, eps) * w[f"{p}.q.norm"], m.get("rot"))
    k = rotate(rms(k, eps) * w[f"{p}.k.norm"], m.get("rot"))
    out = torch.zeros(T, H, Dv, dtype=x.dtype)
    causal = torch.ones(T, T, dtype=torch.bool).tril()
    for h in range(H):
        g = h // (H // G)
        score = (q[:, h] @ k[:, g].T) * float(m["scale"])
        out[:, h] = torch.softmax(score.masked_fill(~causal, -math.inf), -1) @ v[:, g]
    return out.reshape(T, H * Dv) @ w[f"{p}.o"].T


# ----------------------------------------------------------------------------------------------- experts
def relu_square(z: torch.Tensor) -> torch.Tensor:
    return torch.clamp(z, min=0) ** 2


def router_sizes(r: dict):
    """(experts with tensors, identity experts, top, groups, keep)"""
    g = r.get("groups") or {}
    return int(r["experts"]), int(r.get("identity", 0)), int(r["top"]), int(g.get("count", 1)), int(g.get("keep", 1))


def route(x: torch.Tensor, w: Dict[str, torch.Tensor], p: str, r: dict):
    """(chosen ids [T, top], their weights): softmax over all outputs; the choice adds the correction and is confined to the
    groups with the largest single choice score; the weights do neither and are not divided by their sum"""
    E, ident, top, count, keep = router_sizes(r)
    s = torch.softmax(x @ w[f"{p}.router"].T, -1)
    choice = s + w[f"{p}.correction"]
    per = (E + ident) // count
    ids, wts = [], []
    for t in range(x.shape[0]):
        best = [max(float(choice[t, g * per + j]) for j in range(per)) for g in range(count)]
        kept = sorted(range(count), key=lambda g: (-best[g], g))[:keep]
        allowed = [e for g in kept for e in range(g * per, (g + 1) * per)]
        row = sorted(allowed, key=lambda e: (-float(choice[t, e]), e))[:top]
        ids.append(row)
        wts.append([s[t, e] for e in row])
    return torch.tensor(ids), torch.stack([torch.stack(row) for row in wts])


def expert(x: torch.Tensor, w: Dict[str, torch.Tensor], p: str) -> torch.Tensor:
    return relu_square(x @ w[f"{p}.up"].T) @ w[f"{p}.down"].T


def shared_expert(x: torch.Tensor, w: Dict[str, torch.Tensor], p: str) -> torch.Tensor:
    return torch.sigmoid(x @ w[f"{p}.sg"].T) * expert(x, w, p)


def moe(x: torch.Tensor, w: Dict[str, torch.Tensor], p: str, spec: dict) -> torch.Tensor:
    E = int(spec["router"]["experts"])
    ids, wts = route(x, w, p, spec["router"])
    out = torch.zeros_like(x)
    for t in range(x.shape[0]):
        for e, a in zip(ids[t].tolist(), wts[t]):
            out[t] += a * (expert(x[t:t + 1], w, f"{p}.e{e}")[0] if e < E else x[t])
    if spec.get("shared"):
        out = out + shared_expert(x, w, f"{p}.shared")
    return out


# ----------------------------------------------------------------------------------------------- model
def weight_owner(layers: List[dict], i: int) -> int:
    while layers[i].get("weights_of") is not None:
        i = int(layers[i]["weights_of"])
    return i


def forward(tokens: List[int], w: Dict[str, torch.Tensor], cfg: dict, capture: Optional[list] = None,
            last_only: bool = False) -> torch.Tensor:
    """logits [T, vocab] of one sequence ([1, vocab] with ``last_only``); ``capture`` collects the stream after every layer"""
    eps, a = float(cfg["norm"]["eps"]), float(cfg["postln_alpha"])
    x = w["embed"][torch.tensor(tokens)]
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{weight_owner(cfg['layers'], i)}"
        x = shifted_norm(a * x + w[f"{p}.ls1"] * attention(x, w, f"{p}.mix", layer["mixer"], eps), w[f"{p}.norm1"], eps)
        if layer.get("mlp"):
            x = shifted_norm(a * x + w[f"{p}.ls2"] * moe(x, w, f"{p}.mlp", layer["mlp"]), w[f"{p}.norm2"], eps)
        if capture is not None:
            capture.append(x.clone())
    if last_only:
        x = x[-1:]
    return shifted_norm(x, w["final.norm"], eps) @ w["head"].T


# ----------------------------------------------------------------------------------------------- random weights
def tensor_shapes(cfg: dict) -> Dict[str, tuple]:
    W, V = int(cfg["width"]), int(cfg["vocab"])
    out = {"embed": (V, W), "head": (V, W), "final.norm": (W,)}
    for i, layer in enumerate(cfg["layers"]):
        if layer.get("weights_of") is not None:
            continue
        p, m = f"l{i}", layer["mixer"]
        H, G, D, Dv = (int(m[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
        out.update({f"{p}.norm1": (W,), f"{p}.ls1": (W,), f"{p}.mix.q": (H * D, W), f"{p}.mix.q.b": (H * D,),
                    f"{p}.mix.k": (G * D, W), f"{p}.mix.k.b": (G * D,), f"{p}.mix.q.norm": (D,), f"{p}.mix.k.norm": (D,),
                    f"{p}.mix.o": (W, H * Dv)})
        mlp = layer.get("mlp")
        if not mlp:
            continue
        E, ident = router_sizes(mlp["router"])[:2]
        ff = int(mlp["expert"]["ff"])
        out.update({f"{p}.norm2": (W,), f"{p}.ls2": (W,), f"{p}.mlp.router": (E + ident, W), f"{p}.mlp.correction": (E + ident,)})
        for e in range(E):
            out.update({f"{p}.mlp.e{e}.up": (ff, W), f"{p}.mlp.e{e}.down": (W, ff)})
        if mlp.get("shared"):
            sf = int(mlp["shared"]["ff"])
            out.update({f"{p}.mlp.shared.up": (sf, W), f"{p}.mlp.shared.down": (W, sf), f"{p}.mlp.shared.sg": (1, W)})
    return out


def random_weights(cfg: dict, seed: int, dtype=torch.float64) -> Dict[str, torch.Tensor]:
    """weights of a scale at which every mechanism reaches the logits, already rounded to bfloat16 (checkpoints hold that)"""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        z = torch.randn(*shape, generator=g, dtype=torch.float64)
        leaf = name.rsplit(".", 1)[-1]
        if name.endswith((".q.norm", ".k.norm")):
            z = 1.0 + 0.3 * z
        elif leaf in ("norm1", "norm2", "norm"):
            z = 0.2 * z
        elif leaf in ("ls1", "ls2"):
            z = 1.5 + 0.5 * z
        elif leaf == "b":
            z = 0.5 * z
        elif leaf == "correction":
            z = 0.15 * z - 0.2                                     # (choice scores of either sign)
        elif leaf == "router":
            z = 1.5 * z / math.sqrt(shape[-1])
        elif leaf != "embed":
            z = z / math.sqrt(shape[-1])
        out[name] = z.to(torch.bfloat16).to(dtype)
    return out
