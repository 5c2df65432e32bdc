"""Danipel: a pre-norm decoder whose residual is several parallel streams joined by
hyper-connections, with a statistics-free tanh norm and two kinds of latent attention, in whatever
order the configuration lists the layers.

* residual       S fp32 streams per token (``layers.hyper_connection.HyperConnection``): a sublayer
                 reads a learned combination of them, its output is written back to each with a
                 learned weight while the streams are mixed among each other; the streams start as
                 equal copies of the scaled embedding row and are summed at the end;
* norm           ``layers.layernorm.DynamicTanh``: tanh(alpha x) * w + b;
* ``latent_attention``    queries straight from the input, interleaved rotation with YaRN
                 frequencies, a learned sink in the softmax denominator;
* ``latent_attention_2``  queries through a normed low-rank latent, half-split rotation, ordinary
                 softmax; both are ``layers.attention.LatentAttention``: one cached latent and one
                 rotated key part per token, keys and values never expanded;
* feed-forward   dense gated with the tanh form of gelu, or
                 ``layers.moe.CorrectedRoutedExperts`` (choice by corrected scores, identity
                 experts, clamped experts, a shared expert), or none.

Everything that reads a mixer's normed input is ONE projection (``in_proj``).  The stream update,
the next sublayer's read and its norm are one kernel (``ops.hyper_update_norm``), which also adds
the identity experts' share.  Output: the tanh norm of the summed streams and an untied head.

``DanipelConfig.from_dict`` reads the family's ``config.json``.  Single rank only.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

import torch
import torch.nn as nn
import torch.nn.functional as F

from minivllm_amd import ops
from minivllm_amd.layers.activation import GeluTanhAndMul
from minivllm_amd.layers.attention import LatentAttention
from minivllm_amd.layers.hyper_connection import MAX_STREAMS, HyperConnection
from minivllm_amd.layers.layernorm import DynamicTanh
from minivllm_amd.layers.moe import CorrectedRoutedExperts
from minivllm_amd.layers.rotary_embedding import HalfRotation, NeighbourRotation
from minivllm_amd.utils.context import get_context

MIXER_TYPES = ("latent_attention", "latent_attention_2")
EXPERT_SLOPE = 1.702            # the experts' activation is g sigmoid(1.702 g) (u + 1)


# ------------------------------------------------------------------ configuration
@dataclass
class DanipelLayerSpec:
    type: str
    mixer: Dict[str, Any]
    mlp: Optional[Dict[str, Any]]


@dataclass
class DanipelConfig:
    vocab_size: int
    hidden_size: int
    layers: List[DanipelLayerSpec] = field(default_factory=list)
    streams: Optional[int] = None        # None: an ordinary residual sum, no connection tensors
    residual_mult: float = 1.0
    rms_norm_epsilon: float = 1e-6       # of the latents' norms
    embedding_scale: float = 1.0
    max_position: int = 1 << 20          # no table depends on it: positions enter as fp32 angles
    name: str = "danipel"
    architecture: str = "danipel"
    tie_word_embeddings: bool = False

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    @classmethod
    def from_dict(cls, c: dict, name: str = "danipel") -> "DanipelConfig":
        layers = []
        for L in c["layers"]:
            if L["type"] not in MIXER_TYPES:
                raise ValueError(f"unknown layer type {L['type']!r}")
            f = L.get("mlp")
            if f and f.get("kind") not in ("dense", "moe"):
                raise ValueError(f"unknown feed-forward kind {f.get('kind')!r}")
            layers.append(DanipelLayerSpec(L["type"], L["mixer"], f or None))
        streams = c.get("streams")
        return cls(vocab_size=int(c["vocab"]), hidden_size=int(c["width"]), layers=layers,
                   streams=int(streams) if streams is not None else None,
                   residual_mult=float(c.get("residual_mult", 1.0)),
                   rms_norm_epsilon=float(c["norm"]["eps"]),
                   embedding_scale=float((c.get("embedding") or {}).get("scale", 1.0)),
                   max_position=int(c.get("max_position", 1 << 20)), name=name)

    def validate_engine(self, engine_cfg) -> None:
        if engine_cfg.tp_degree != 1:
            raise ValueError("Danipel runs on one rank (its mixers are not sharded)")
        if self.streams is not None and not 1 <= self.streams <= MAX_STREAMS:
            raise ValueError(f"streams must lie in 1 .. {MAX_STREAMS}")
        for L in self.layers:
            m = L.mixer
            if int(m["rot"]["dims"]) > int(m["rot_dim"]) or int(m["rot"]["dims"]) % 2:
                raise ValueError("rot.dims must be even and at most rot_dim")
            if int(m["kv_rank"]) + int(m["rot_dim"]) > 1024:
                raise ValueError("attention over the latent runs with key rows of at most 1024 "
                                 "numbers (kv_rank + rot_dim)")
            f = L.mlp
            if f and f["kind"] == "moe":
                r = f["router"]
                if not 0 < int(r["top"]) <= int(r["experts"]) + int(r.get("identity", 0)):
                    raise ValueError("router: `top` must lie in 1 .. experts + identity")


def _param(t: torch.Tensor, like: torch.Tensor) -> nn.Parameter:
    return nn.Parameter(t.to(device=like.device, dtype=like.dtype).contiguous(), requires_grad=False)


def _take(w: dict, key: str, shape, where: str) -> torch.Tensor:
    if key not in w:
        raise KeyError(f"checkpoint lacks {where}{key}")
    t = w.pop(key)
    if tuple(t.shape) != tuple(shape):
        raise ValueError(f"shape mismatch for {where}{key}: expected {tuple(shape)}, checkpoint "
                         f"has {tuple(t.shape)}")
    return t


def _load_norm(norm: DynamicTanh, w: dict, name: str, where: str) -> None:
    W = norm.weight.shape[0]
    norm.weight.copy_(_take(w, name, (W,), where))
    norm.bias.copy_(_take(w, name + ".b", (W,), where))
    norm.alpha.copy_(_take(w, name + ".alpha", (), where).reshape(1))


def _norm_shapes(name: str, W: int):
    return [(name, (W,)), (name + ".b", (W,)), (name + ".alpha", ())]


def _up8(n: int) -> int:
    return n + (-n % 8)


# ------------------------------------------------------------------ mixers
class DanipelLatentMixer(nn.Module):
    """Both kinds of latent attention; ``low_rank`` (the second kind): queries through a normed
    latent of their own, half-split rotation, no sink."""

    def __init__(self, W: int, kind: str, m: dict, eps: float):
        super().__init__()
        self.W, self.eps, self.low_rank = W, eps, kind == "latent_attention_2"
        H, D, P, E, R = (int(m[k]) for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
        rot = (HalfRotation if self.low_rank else NeighbourRotation)(
            int(m["rot"]["dims"]), float(m["rot"]["base"]), m["rot"].get("scaling"))
        self.attn = LatentAttention(H, D, P, E, R, float(m["scale"]), 0, rot, eps, sink=not self.low_rank)
        self.q_cols = int(m["q_rank"]) if self.low_rank else H * (D + P)
        if self.low_rank:
            self.q_norm = nn.Parameter(torch.ones(self.q_cols, dtype=torch.float32), requires_grad=False)
            self.up_q = nn.Parameter(torch.zeros(H * (D + P), self.q_cols), requires_grad=False)
        # q's rows, padded so that the latent's block starts on a run of eight columns
        self.in_proj = nn.Parameter(torch.zeros(1, W), requires_grad=False)
        self.o_proj = nn.Parameter(torch.zeros(W, H * E), requires_grad=False)

    def attention_cores(self):
        return [self.attn.core]

    def forward(self, h: torch.Tensor) -> torch.Tensor:
        a = self.attn
        T, at = h.shape[0], _up8(self.q_cols)
        proj = F.linear(h, self.in_proj)
        q, dkv = proj[:, :self.q_cols], proj[:, at:at + a.kv_rank + a.rot_dim]
        if self.low_rank:
            q = F.linear(ops.rms_norm_rows(q, self.q_norm, self.eps, h.dtype), self.up_q)
        o = a(q.view(T, a.num_heads, a.head_dim + a.rot_dim), dkv)
        return F.linear(o.view(T, -1), self.o_proj)

    def load(self, w: dict, where: str, like) -> None:
        W, a, Q = self.W, self.attn, self.q_cols
        H, D, P, E, R = a.num_heads, a.head_dim, a.rot_dim, a.v_head_dim, a.kv_rank
        rows = [_take(w, "dq" if self.low_rank else "q", (Q, W), where)]
        if _up8(Q) > Q:
            rows.append(torch.zeros(_up8(Q) - Q, W, dtype=rows[0].dtype))
        rows.append(_take(w, "dkv", (R + P, W), where))
        if (R + P) % 8:                                  # row stride of the output: whole runs of 8
            rows.append(torch.zeros(-(R + P) % 8, W, dtype=rows[0].dtype))
        self.in_proj = _param(torch.cat(rows, 0), like)
        if self.low_rank:
            self.q_norm.copy_(_take(w, "dq.norm", (Q,), where))
            self.up_q = _param(_take(w, "uq", (H * (D + P), Q), where), like)
        else:
            a.core.sink.copy_(_take(w, "sink", (H,), where))
        a.latent_norm.copy_(_take(w, "dkv.norm", (R,), where))
        a.load_expansions(_take(w, "uk", (H * D, R), where), _take(w, "uv", (H * E, R), where), like)
        self.o_proj = _param(_take(w, "o", (W, H * E), where), like)

    @staticmethod
    def shapes(W, kind, m):
        H, D, P, E, R = (int(m[k]) for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
        if kind == "latent_attention_2":
            Q = int(m["q_rank"])
            out = [("dq", (Q, W)), ("dq.norm", (Q,)), ("uq", (H * (D + P), Q))]
        else:
            out = [("q", (H * (D + P), W)), ("sink", (H,))]
        return out + [("dkv", (R + P, W)), ("dkv.norm", (R,)), ("uk", (H * D, R)), ("uv", (H * E, R)),
                      ("o", (W, H * E))]


# ------------------------------------------------------------------ feed-forward
# ``forward(h)`` returns (output [T, W], what ``ops.hyper_update_norm`` adds besides it, or None).
class DanipelDenseFF(nn.Module):
    def __init__(self, W: int, f: dict):
        super().__init__()
        self.W, self.ff = W, int(f["ff"])
        self.act = GeluTanhAndMul()
        self.gate_up = nn.Parameter(torch.zeros(2 * self.ff, W), requires_grad=False)
        self.down = nn.Parameter(torch.zeros(W, self.ff), requires_grad=False)

    def forward(self, h):
        return F.linear(self.act(F.linear(h, self.gate_up)), self.down), None

    def load(self, w: dict, where: str, like) -> None:
        W, n = self.W, self.ff
        self.gate_up = _param(torch.cat([_take(w, k, (n, W), where) for k in ("gate", "up")], 0), like)
        self.down = _param(_take(w, "down", (W, n), where), like)

    @staticmethod
    def shapes(W, f):
        n = int(f["ff"])
        return [("gate", (n, W)), ("up", (n, W)), ("down", (W, n))]


class DanipelRoutedFF(CorrectedRoutedExperts):
    def __init__(self, W: int, f: dict):
        r, sh = f["router"], f.get("shared") or {}
        super().__init__(W, int(f["expert"]["ff"]), int(r["experts"]), int(r.get("identity", 0)),
                         int(r["top"]), float(f["expert"]["limit"]), float(r.get("scale", 1.0)),
                         int(sh.get("ff", 0)), float(sh.get("limit", 0.0)), slope=EXPERT_SLOPE)
        self.W = W

    def load(self, w: dict, where: str, like) -> None:
        W = self.W
        names = [(f"e{e}.", self.ff) for e in range(self.experts)]
        names += [("shared.", self.shared_ff)] if self.shared_ff else []
        gates = [_take(w, n + "gate", (s, W), where) for n, s in names]
        ups = [_take(w, n + "up", (s, W), where) for n, s in names]
        self.gate_up = _param(torch.cat(gates + ups, 0), like)
        self.down = _param(torch.cat([_take(w, n + "down", (W, s), where) for n, s in names], 1), like)
        rows = self.experts + self.identity
        self.router.copy_(_take(w, "router", (rows, W), where))
        self.correction.copy_(_take(w, "correction", (rows,), where))

    @staticmethod
    def shapes(W, f):
        r = f["router"]
        names = [(f"e{e}.", int(f["expert"]["ff"])) for e in range(int(r["experts"]))]
        names += [("shared.", int(f["shared"]["ff"]))] if f.get("shared") else []
        rows = int(r["experts"]) + int(r.get("identity", 0))
        out = []
        for n, s in names:
            out += [(n + "gate", (s, W)), (n + "up", (s, W)), (n + "down", (W, s))]
        return out + [("router", (rows, W)), ("correction", (rows,))]


_FEED_FORWARDS = {"dense": DanipelDenseFF, "moe": DanipelRoutedFF}


# ------------------------------------------------------------------ layers
class DanipelSublayer(nn.Module):
    """A norm, what it feeds (mixer or feed-forward) and the connection to the streams."""

    def __init__(self, cfg: DanipelConfig, body: nn.Module, prefix: str, number: int):
        super().__init__()
        self.norm = DynamicTanh(cfg.hidden_size)
        self.body = body
        self.connection = HyperConnection(cfg.streams or 1, cfg.residual_mult)
        self.learned_connection = cfg.streams is not None
        self.prefix, self.number = prefix, number

    def forward(self, h: torch.Tensor):
        """The normed input -> (output, what joins it in the stream update)."""
        y = self.body(h)
        return y if isinstance(y, tuple) else (y, None)

    def load(self, w: dict, where: str, like) -> None:
        _load_norm(self.norm, w, f"norm{self.number}", where)
        part = {k[len(self.prefix):]: w.pop(k) for k in [k for k in w if k.startswith(self.prefix)]}
        self.body.load(part, where + self.prefix, like)
        if part:
            raise KeyError(f"checkpoint tensor {where}{self.prefix}{next(iter(part))} has no parameter")
        if self.learned_connection:
            s, hc = self.connection.streams, f"hc{self.number}."
            self.connection.load(_take(w, hc + "in", (s,), where), _take(w, hc + "out", (s,), where),
                                 _take(w, hc + "mix", (s, s), where))


class DanipelLayer(nn.Module):
    def __init__(self, cfg: DanipelConfig, spec: DanipelLayerSpec):
        super().__init__()
        W = cfg.hidden_size
        self.kind = spec.type
        self.mix = DanipelLatentMixer(W, spec.type, spec.mixer, cfg.rms_norm_epsilon)
        subs = [DanipelSublayer(cfg, self.mix, "mix.", 1)]
        if spec.mlp:
            subs.append(DanipelSublayer(cfg, _FEED_FORWARDS[spec.mlp["kind"]](W, spec.mlp), "mlp.", 2))
        self.sublayers = nn.ModuleList(subs)

    def load(self, w: dict, where: str, like) -> None:
        for s in self.sublayers:
            s.load(w, where, like)
        if w:
            raise KeyError(f"checkpoint tensor {where}{next(iter(w))} has no parameter")


class DanipelModel(nn.Module):
    def __init__(self, cfg: DanipelConfig):
        super().__init__()
        self.embed = nn.Embedding(cfg.vocab_size, cfg.hidden_size)
        self.embed.weight.requires_grad_(False)
        self.embed_scale = cfg.embedding_scale
        self.streams = cfg.streams or 1
        self.layers = nn.ModuleList([DanipelLayer(cfg, s) for s in cfg.layers])
        self.act_dtype = self.embed.weight.dtype
        # observer for tests: called with (layer index, sum of the streams) after every layer
        self.layer_hook = None

    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor) -> torch.Tensor:
        """Returns the fp32 streams [T, S, W] after the last layer (their sum and the final norm
        belong to the head: only the rows whose logits are wanted go through them)."""
        dt = self.act_dtype
        x0 = ops.embed_sum(input_ids, None, self.embed.weight, None, self.embed_scale)
        # until the first update the S streams are one row seen S times
        x = x0[:, None, :].expand(-1, self.streams, -1)
        todo = [(i, sub) for i, layer in enumerate(self.layers) for sub in layer.sublayers]
        h = None
        if todo:
            first = todo[0][1]
            h = ops.hyper_norm(x, first.connection.read, first.norm.parts, dt)
        for n, (i, sub) in enumerate(todo):
            y, skip = sub(h)
            nxt = todo[n + 1][1] if n + 1 < len(todo) else None
            c = sub.connection
            x, h = ops.hyper_update_norm(x, y, skip, c.write, c.mix,
                                         nxt.connection.read if nxt else None,
                                         nxt.norm.parts if nxt else None, dt)
            if self.layer_hook is not None and (nxt is None or todo[n + 1][0] != i):
                self.layer_hook(i, x.sum(1))
        return x


class SummedStreamsHead(nn.Module):
    """Sum of the streams, final tanh norm and untied output projection, applied to the rows a step
    wants (each sequence's last row, or the context's ``logit_rows``)."""

    def __init__(self, vocab_size: int, hidden_size: int, streams: int):
        super().__init__()
        self.norm = DynamicTanh(hidden_size)
        self.register_buffer("ones", torch.ones(streams, dtype=torch.float32), persistent=False)
        self.weight = nn.Parameter(torch.zeros(vocab_size, hidden_size), requires_grad=False)
        self.num_embeddings = vocab_size
        self.vocab_start = 0

    def select_last(self, hidden: torch.Tensor) -> torch.Tensor:
        ctx = get_context()
        if ctx.logit_rows is not None:
            return hidden.index_select(0, ctx.logit_rows.long())
        if ctx.is_prefill and ctx.cu_seqlens_q is not None:
            return hidden.index_select(0, (ctx.cu_seqlens_q[1:] - 1).long())
        return hidden

    def local_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        rows = self.select_last(hidden)
        return F.linear(ops.hyper_norm(rows, self.ones, self.norm.parts, self.weight.dtype), self.weight)

    def forward(self, hidden: torch.Tensor) -> torch.Tensor:
        return self.local_logits(hidden)


class DanipelForCausalLM(nn.Module):
    needs_aux_rows = False
    has_recurrent_state = False
    prefix_cacheable = True         # one latent row per token and layer, a function of the prefix alone

    def __init__(self, config: DanipelConfig):
        super().__init__()
        self.config = config
        self.model = DanipelModel(config)
        self.lm_head = SummedStreamsHead(config.vocab_size, config.hidden_size, config.streams or 1)

    def forward(self, input_ids, positions=None):
        if positions is None:
            positions = get_context().positions
        return self.model(input_ids, positions)

    def compute_logits(self, hidden):
        return self.lm_head(hidden)

    def compute_local_logits(self, hidden):
        return self.lm_head.local_logits(hidden)

    # ---- what the engine needs to know about caches and state ---------------------------
    def attention_layers(self):
        return [a for l in self.model.layers for a in l.mix.attention_cores()]

    def state_layers(self):
        return []

    # ---- weights -----------------------------------------------------------------------
    @torch.no_grad()
    def load_weights(self, items) -> int:
        """``items``: iterable of (checkpoint name, tensor).  The tensors of a layer are collected
        and then stacked into its fused parameters; unknown, missing or mis-shaped tensors raise
        with their name."""
        like = self.model.embed.weight
        per_layer: List[dict] = [dict() for _ in self.model.layers]
        top: Dict[str, torch.Tensor] = {}
        n = 0
        for name, t in items:
            n += 1
            li, _, rest = name.partition(".")
            if li.startswith("l") and li[1:].isdigit() and int(li[1:]) < len(per_layer):
                per_layer[int(li[1:])][rest] = t
            else:
                top[name] = t
        like.copy_(_take(top, "embed", like.shape, ""))
        self.lm_head.weight.copy_(_take(top, "head", self.lm_head.weight.shape, ""))
        _load_norm(self.lm_head.norm, top, "final.norm", "")
        if top:
            raise KeyError(f"checkpoint tensor {next(iter(top))!r} has no parameter")
        for i, (layer, w) in enumerate(zip(self.model.layers, per_layer)):
            layer.load(w, f"l{i}.", like)
        return n

    def checkpoint_shapes(self):
        """(name, shape) of every tensor a checkpoint of this configuration holds."""
        c = self.config
        W = c.hidden_size
        yield "embed", (c.vocab_size, W)
        for i, L in enumerate(c.layers):
            p = f"l{i}."
            parts = [("mix.", DanipelLatentMixer.shapes(W, L.type, L.mixer))]
            if L.mlp:
                parts.append(("mlp.", _FEED_FORWARDS[L.mlp["kind"]].shapes(W, L.mlp)))
            for q, (prefix, shapes) in enumerate(parts, 1):
                for nm, shape in _norm_shapes(f"norm{q}", W):
                    yield p + nm, shape
                for nm, shape in shapes:
                    yield p + prefix + nm, shape
                if c.streams is not None:
                    s = c.streams
                    yield p + f"hc{q}.in", (s,)
                    yield p + f"hc{q}.out", (s,)
                    yield p + f"hc{q}.mix", (s, s)
        for nm, shape in _norm_shapes("final.norm", W):
            yield nm, shape
        yield "head", (c.vocab_size, W)

    def random_checkpoint(self, seed: int = 0):
        """Seeded random tensors (values exactly representable in bfloat16) of every checkpoint
        name, scaled so that activations stay O(1) through the stack."""
        g = torch.Generator().manual_seed(seed)
        S = self.config.streams or 1
        out = {}
        for name, shape in self.checkpoint_shapes():
            leaf = name.rsplit(".", 1)[-1]
            r = torch.randn(shape, generator=g)
            if leaf.startswith("norm"):
                t = 1.0 + 0.1 * r
            elif leaf in ("b", "correction"):
                t = 0.05 * r
            elif leaf == "alpha":
                t = 0.7 + 0.1 * r
            elif leaf == "sink":
                t = 0.5 * r
            elif leaf == "in":
                t = (1.0 + 0.2 * r) / S
            elif leaf == "out":
                t = 1.0 + 0.2 * r
            elif leaf == "mix":
                t = torch.eye(S) * 0.9 + 0.1 / S + 0.05 * r
            elif name == "embed":
                t = r / max(self.config.embedding_scale, 1e-6)
            elif leaf in ("down", "o"):
                t = 0.5 * r * (shape[-1] ** -0.5)
            else:
                t = r * (shape[-1] ** -0.5)
            out[name] = t.to(torch.bfloat16)
        return out

    def init_random_weights(self, seed: int = 0, std: float = 0.02) -> None:
        self.load_weights(self.random_checkpoint(seed).items())
