"""Kirenex: a decoder-only design of sequential post-norm sublayers over an fp32 residual stream,
    x <- N(alpha x + mixer(x)) w1;    x <- N(alpha x + ff(x)) w2,
N being division by the row's root mean square and alpha one constant of the model: every sublayer reads the stream itself,
which starts as the token's row plus a learned row of its position.  The mixer is, layer by layer, one of two:
* attention over a latent: the cache holds one normed latent and one rotated key part (interleaved pairs) per token, from which
  every head's unrotated key and value derive; an output gate per element; a layer may attend to the rows another layer made;
* two mixers side by side on the same input, each normed over the model width, averaged: grouped-query softmax attention (q and k
  normed per head with a learned weight, then rotated on part of the head with frequencies rescaled by wavelength; a sliding
  window behind which the first tokens stay visible) and a delta rule with one decay per head (short convolutions, unit keys,
  a silu output gate).
The feed-forward is a gated one with the tanh form of GELU.  Embedding and head are separate tables.

Everything that differs between models of the design comes from config.json (``KirenexConfig``); the model is assembled from
the framework's mechanisms - PostNorm / GluFF / AngleRotary / HalfAngleRotary (layers.py), LatentAttention +
PooledWindowAttention + SequenceBackend (attention.py), HeadDeltaMixer (recurrent.py), WindowKVPool + RecurrentStatePool
(pool.py), LogitsProcessor (llama.py) - and served by the ModelRunner like the other model classes."""
from typing import Iterable, List, Optional, Tuple

import torch
from torch import nn

from . import _native
from .attention import LatentAttention, PooledWindowAttention
from .forward_info import ForwardBatch
from .layers import AngleRotary, GluFF, GroupRMSNorm, HalfAngleRotary, PostNorm
from .llama import LogitsProcessor, LogitsProcessorOutput, ParallelLMHead
from .recurrent import HeadDeltaMixer

MIXERS = ("latent_attention", "parallel")


class KirenexConfig:
    """config.json of the design, plus what the runner asks of any model configuration (vocab_size, context_len,
    num_hidden_layers, is_encoder_decoder) and what it builds the pools from.  The learned position rows bound the context."""
    architecture = "Kirenex"
    is_encoder_decoder = False
    vision_config = None
    tie_word_embeddings = False

    def __init__(self, raw: dict, context_len: Optional[int] = None):
        self.raw = raw
        self.vocab_size = int(raw["vocab"])
        self.hidden_size = int(raw["width"])
        self.layers: List[dict] = raw["layers"]
        self.num_hidden_layers = len(self.layers)
        self.rms_norm_eps = float(raw["norm"]["eps"])
        self.alpha = float(raw["postln_alpha"])
        self.max_positions = int(raw["max_positions"])
        self.context_len = min(context_len or self.max_positions, self.max_positions)
        for i, layer in enumerate(self.layers):
            if layer["type"] not in MIXERS:
                raise ValueError(f"unknown layer type {layer['type']!r}")
            if layer.get("mlp") is not None and layer["mlp"]["kind"] != "dense":
                raise ValueError(f"unknown feed-forward kind {layer['mlp']['kind']!r}")
            if layer["type"] == "latent_attention" and layer["mixer"].get("kv_from") is not None:
                m, j = layer["mixer"], int(layer["mixer"]["kv_from"])
                if not 0 <= j < i or self.layers[j]["type"] != "latent_attention" or self.layers[j]["mixer"].get("kv_from") is not None:
                    raise ValueError("kv_from must name an earlier latent attention layer that makes its own rows")
                if any(m[k] != self.layers[j]["mixer"][k] for k in ("kv_rank", "rot_dim", "rot")):
                    raise ValueError("layers that share latent rows must agree on kv_rank, rot_dim and rot")

    # ---- what the runner builds its pools from
    def window_cache(self):
        """{layer id: (kv_heads, dim, vdim, pooled)} of the layers that keep a key/value row per token"""
        return {i: (int(l["mixer"]["left"]["kv_heads"]), int(l["mixer"]["left"]["dim"]), int(l["mixer"]["left"]["vdim"]), False)
                for i, l in enumerate(self.layers) if l["type"] == "parallel"}

    def latent_cache(self):
        """{layer id: (rank, rot_dim)} of the layers that keep a latent row per token"""
        return {i: (int(l["mixer"]["kv_rank"]), int(l["mixer"]["rot_dim"])) for i, l in enumerate(self.layers)
                if l["type"] == "latent_attention" and l["mixer"].get("kv_from") is None}

    def shift_layers(self):
        return []                                     # no mixer reads the previous token's input

    def named_state(self):
        """{layer id: {name: shape}} of the fp32 state the recurrent mixers carry per request"""
        out = {}
        for i, l in enumerate(self.layers):
            if l["type"] == "parallel":
                r = l["mixer"]["right"]
                out[i] = HeadDeltaMixer.state_shapes(int(r["heads"]), int(r["kv_heads"]), int(r["dim"]), int(r["vdim"]), int(r["conv"]))
        return out

    def cache_bytes_per_token(self, kv_dtype: torch.dtype) -> int:
        per = sum(g * (d + dv) for g, d, dv, _ in self.window_cache().values()) + sum(r + d for r, d in self.latent_cache().values())
        return max(1, per * torch.finfo(kv_dtype).bits // 8)


class KirenexLatentAttention(nn.Module):
    """ONE product makes the rows [q | latent and key part | gate] (a layer that reads another layer's rows: [q | gate]); the
    up-projections of keys and values are folded into the query and the output, a product per head on either side."""

    def __init__(self, width: int, m: dict, layer_id: int, eps: float, dtype=None):
        super().__init__()
        H, D, R, Dv, C = (int(m[k]) for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
        self.heads, self.dim, self.rot_dim, self.vdim, self.rank, self.eps = H, D, R, Dv, C, eps
        self.own = m.get("kv_from") is None
        self.kv_rows = C + R if self.own else 0
        self.in_proj = nn.Parameter(torch.empty(H * (D + R) + self.kv_rows + H * Dv, width, dtype=dtype), requires_grad=False)
        self.latent_norm = nn.Parameter(torch.ones(C, dtype=torch.float32), requires_grad=False) if self.own else None
        self.uk_t = nn.Parameter(torch.empty(H, C, D, dtype=dtype), requires_grad=False)     # per head [rank, dim]
        self.uv = nn.Parameter(torch.empty(H, Dv, C, dtype=dtype), requires_grad=False)      # per head [vdim, rank]
        self.o = nn.Parameter(torch.empty(width, H * Dv, dtype=dtype), requires_grad=False)
        rot = m["rot"]
        if int(rot["dims"]) > R:
            raise ValueError("rot.dims exceeds rot_dim")
        self.rotary = AngleRotary(int(rot["dims"]), float(rot["base"]), rot.get("scaling"))
        self.attn = LatentAttention(H, C, R, float(m["scale"]), layer_id if self.own else int(m["kv_from"]))

    def forward(self, positions, h: torch.Tensor, forward_batch: ForwardBatch) -> torch.Tensor:
        H, D, R = self.heads, self.dim, self.rot_dim
        nq = H * (D + R)
        a = _native.linear(h, self.in_proj)
        q = a[:, :nq].view(h.shape[0], H, D + R)
        self.attn.store(a[:, nq:nq + self.kv_rows] if self.own else None, None if self.latent_norm is None else self.latent_norm.data,
                        q, D, self.rotary, positions, self.eps, forward_batch)
        q_lat = _native.head_linear(q[:, :, :D], self.uk_t)                                    # [T, H, rank]
        o_lat = self.attn(q_lat, q[:, :, D:], forward_batch, token_major=True)
        o = _native.head_linear(o_lat, self.uv, gate=a[:, nq + self.kv_rows:])                 # [T, H, vdim]
        return _native.linear(o.view(h.shape[0], H * self.vdim), self.o)


class KirenexParallel(nn.Module):
    """Two mixers on the same input: windowed softmax attention (left) and a head-gated delta rule (right).  ONE product makes
    the rows [q | k | v (left) | q | k | v | g (right)]; the two results go back separately (the layer norms each over the model
    width and averages them)."""

    def __init__(self, width: int, m: dict, layer_id: int, eps: float, dtype=None):
        super().__init__()
        a, b = m["left"], m["right"]
        H, G, D, Dv = (int(a[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
        self.heads, self.kv_heads, self.dim, self.vdim, self.eps = H, G, D, Dv, eps
        self.left_rows = H * D + G * D + G * Dv
        self.right = HeadDeltaMixer(width, int(b["heads"]), int(b["kv_heads"]), int(b["dim"]), int(b["vdim"]), int(b["conv"]), eps,
                                    layer_id=layer_id, own_input=False, dtype=dtype)
        self.in_proj = nn.Parameter(torch.empty(self.left_rows + self.right.in_rows, width, dtype=dtype), requires_grad=False)
        self.left_o = nn.Parameter(torch.empty(width, H * Dv, dtype=dtype), requires_grad=False)
        rot = a.get("rot")
        self.rotary = None
        if rot and int(rot["dims"]) > 0:
            if int(rot["dims"]) > D:
                raise ValueError("rot.dims exceeds the head size")
            self.rotary = HalfAngleRotary(int(rot["dims"]), float(rot["base"]), rot.get("scaling"))
        mask = a.get("mask") or {}
        self.attn = PooledWindowAttention(H, G, D, Dv, float(a["scale"]), layer_id, window=mask.get("size"), norm_values=False,
                                          qk_norm="before", keep_first=int(mask.get("keep_first") or 0))

    def forward(self, positions, x: torch.Tensor, h: torch.Tensor, forward_batch: ForwardBatch):
        nq, nk = self.heads * self.dim, self.kv_heads * self.dim
        a = _native.linear(h, self.in_proj)
        q = a[:, :nq]
        self.attn.store(q, a[:, nq:nq + nk], a[:, nq + nk:self.left_rows], self.rotary, positions, self.eps, forward_batch)
        left = _native.linear(self.attn(q, forward_batch), self.left_o)
        return left, self.right.scan(a[:, self.left_rows:], x, forward_batch)


class KirenexLayer(nn.Module):
    def __init__(self, config: KirenexConfig, layer_id: int, dtype=None):
        super().__init__()
        spec, W, eps = config.layers[layer_id], config.hidden_size, config.rms_norm_eps
        self.kind = spec["type"]
        self.mix = (KirenexParallel if self.kind == "parallel" else KirenexLatentAttention)(W, spec["mixer"], layer_id, eps, dtype)
        self.norm1 = PostNorm(W, eps, config.alpha, branches=2 if self.kind == "parallel" else 1)
        self.mlp = None
        if spec.get("mlp") is not None:
            self.mlp = GluFF(W, int(spec["mlp"]["ff"]), "gelu_tanh", dtype=dtype)
            self.norm2 = PostNorm(W, eps, config.alpha)

    def forward(self, positions, x: torch.Tensor, h: torch.Tensor, forward_batch: ForwardBatch, dtype,
                want_lo: bool) -> Optional[torch.Tensor]:
        """x: the fp32 stream, updated in place; h = x in the projections' dtype.  Returns the new x in that dtype."""
        y = self.mix(positions, x, h, forward_batch) if self.kind == "parallel" else self.mix(positions, h, forward_batch)
        if self.mlp is None:
            return self.norm1(x, y, dtype, want_lo)
        h = self.norm1(x, y, dtype)
        return self.norm2(x, self.mlp(h), dtype, want_lo)


class KirenexForCausalLM(nn.Module):
    # parameters keep the dtypes they are declared with (fp32 norms, decays, gate rows) whatever the runner's dtype
    keeps_parameter_dtypes = True
    supports_tensor_parallel = False
    # Largest decode step that is captured into a HIP graph (the step has no host synchronisation and no data-dependent
    # shape); larger steps run eagerly.
    max_graph_batch = 64
    # sources of the HIP library this model's path needs beyond the core (scratchpad_amd.build.build_native(only=...));
    # ssm.hip: the short convolution and the fp32 product of few rows that gates share
    NATIVE_SOURCES = ["stream_norm.hip", "window_attention.hip", "latent_attention.hip", "head_delta.hip", "ssm.hip"]

    def __init__(self, config: KirenexConfig, dtype=None):
        super().__init__()
        self.config = config
        self.dtype = dtype or torch.get_default_dtype()
        W = config.hidden_size
        self.embed = nn.Parameter(torch.empty(config.vocab_size, W, dtype=dtype), requires_grad=False)
        self.pos = nn.Parameter(torch.empty(config.max_positions, W, dtype=dtype), requires_grad=False)
        self.layers = nn.ModuleList([KirenexLayer(config, i, dtype) for i in range(config.num_hidden_layers)])
        self.norm = GroupRMSNorm(W, 1, config.rms_norm_eps)
        self.lm_head = ParallelLMHead(config.vocab_size, W, dtype)
        self.logits_processor = LogitsProcessor(config)
        self.capture_layers: Optional[list] = None     # set to a list to collect the stream after every layer

    @torch.no_grad()
    def forward(self, input_ids, positions, forward_batch: ForwardBatch, input_embeds=None) -> LogitsProcessorOutput:
        dtype = self.embed.dtype
        x, h = _native.embed_scale(self.embed.data, input_ids, 1.0, want_lo=True, table=self.pos.data, positions=positions)
        last = len(self.layers) - 1
        for i, layer in enumerate(self.layers):
            h = layer(positions, x, h, forward_batch, dtype, i < last)
            if self.capture_layers is not None:
                self.capture_layers.append(x.clone())
        return self.logits_processor(input_ids, self.norm(x, dtype), self.lm_head, forward_batch)

    # ---- weights --------------------------------------------------------------------------------------------------
    def load_weights(self, weights: Iterable[Tuple[str, torch.Tensor]]) -> None:
        """Checkpoint names of the design ('embed', 'pos', 'head', 'final.norm', 'l<i>.norm1|norm2', 'l<i>.mix.*',
        'l<i>.mlp.gate|up|down') -> this module's (partly merged, partly transposed) parameters."""
        w = dict(weights)
        used = set()

        def take(name):
            used.add(name)
            return w[name]

        def put(param: nn.Parameter, value: torch.Tensor):
            value = value.reshape(param.shape) if value.numel() == param.numel() and value.dim() != param.dim() else value
            if value.shape != param.shape:
                raise RuntimeError(f"shape {tuple(value.shape)} does not fit parameter {tuple(param.shape)}")
            param.data.copy_(value.to(param.dtype))

        def rows(prefix, *names):
            return torch.cat([take(f"{prefix}.{n}") for n in names], 0)

        put(self.embed, take("embed"))
        put(self.pos, take("pos"))
        put(self.lm_head.weight, self.lm_head.shard_from_full(take("head")))
        put(self.norm.weight, take("final.norm"))
        for i, layer in enumerate(self.layers):
            p, mix = f"l{i}", layer.mix
            M = f"{p}.mix"
            put(layer.norm1.weight, take(f"{p}.norm1"))
            if layer.kind == "latent_attention":
                H, D, Dv, C = mix.heads, mix.dim, mix.vdim, mix.rank
                put(mix.in_proj, rows(M, "q", "dkv", "g") if mix.own else rows(M, "q", "g"))
                if mix.own:
                    put(mix.latent_norm, take(f"{M}.dkv.norm"))
                put(mix.uk_t, take(f"{M}.uk").view(H, D, C).transpose(1, 2))
                put(mix.uv, take(f"{M}.uv").view(H, Dv, C))
                put(mix.o, take(f"{M}.o"))
            else:
                L, R, right = f"{M}.left", f"{M}.right", mix.right
                put(mix.in_proj, torch.cat([rows(L, "q", "k", "v"), rows(R, "q", "k", "v", "g")], 0))
                put(mix.attn.q_norm, take(f"{L}.q.norm"))
                put(mix.attn.k_norm, take(f"{L}.k.norm"))
                put(mix.left_o, take(f"{L}.o"))
                put(right.gates, rows(R, "b", "a"))
                put(right.conv, rows(R, "q.conv", "k.conv", "v.conv"))
                for name in ("dt_bias", "A_log", "norm", "o"):
                    put(getattr(right, name), take(f"{R}.{name}"))
                put(layer.norm1.branch_weight, torch.stack([take(f"{L}.out"), take(f"{R}.out")]))
            if layer.mlp is not None:
                put(layer.norm2.weight, take(f"{p}.norm2"))
                put(layer.mlp.gate_up, rows(f"{p}.mlp", "gate", "up"))
                put(layer.mlp.down, take(f"{p}.mlp.down"))
        extra = set(w) - used
        if extra:
            import warnings
            warnings.warn(f"checkpoint tensors no part of the configured model reads: {sorted(extra)[:8]}")

    def init_random(self, generator: torch.Generator) -> None:
        """random weights of a plausible scale (benchmarks and tests of the host path: no checkpoint)"""
        for name, p in self.named_parameters():
            leaf = name.rsplit(".", 1)[-1]
            if leaf in ("norm", "latent_norm", "q_norm", "k_norm", "branch_weight") or (leaf == "weight" and p.dim() == 1):
                p.data.fill_(1.0)
            elif leaf in ("embed", "pos"):
                p.data.normal_(0.0, 1.0, generator=generator)
            elif leaf in ("A_log", "dt_bias"):
                p.data.normal_(-1.0, 0.5, generator=generator)
            elif leaf == "conv":
                p.data.normal_(0.0, 0.5, generator=generator)
            else:
                p.data.normal_(0.0, 1.0 / (p.shape[-1] ** 0.5), generator=generator)
