"""Plain float64 restatement of the Danipel decoder, one function per mechanism.  It shares no code
with the package: the tests compare the engine with it.

The design in this file's notation (W = width, s = streams, m = the residual multiplier):

* every token starts s equal copies of E[token] * s_e, the streams x_1 .. x_s;
* a sublayer (a mixer, then a feed-forward, which may be absent) with its own numbers `in` [s],
  `out` [s], `mix` [s, s]: u = sum_a in[a] x_a; y = sublayer(norm u); then, from the old streams,
  x_b <- sum_a mix[a, b] x_a + m out[b] y (mix is indexed [from, to]);
* norm: tanh(alpha u) w + b with one number alpha (no mean, no variance);
* mixers "latent_attention" and "latent_attention_2": c = rmsnorm of the first R rows of W_dkv h
  times a weight, r = the last P rows, turned; head h's key is [W_uk_h c | r], its value W_uv_h c;
  q per head = [D unrotated | P turned]; score = scale (q . k); every earlier position is seen.
  The first kind takes q = W_q h, turns neighbouring pairs with YaRN's frequencies, cos and sin
  both times 0.1 ln(factor) + 1, and has exp(sink_h) in the softmax denominator; the second takes
  q = W_uq rmsnorm(W_dq h), turns half-split pairs with plain frequencies, ordinary softmax;
* feed-forward: dense W_down (gelu_tanh(W_gate h) W_up h), or routed: scores = softmax over the
  experts and the identity experts behind them; the `top` largest score + correction are chosen;
  weights = their scores, divided by their sum, times `scale`; an identity expert returns h;
  expert: g = min(W_gate h, L), u = clamp(W_up h, -L, L), W_down (g sigmoid(1.702 g) (u + 1)); a
  shared expert of the same form is added for every token;
* logits = head norm(sum of the streams).
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def tanh_norm(x, alpha, w, b):
    return torch.tanh(alpha * x) * w + b


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def frequencies(rot):
    """([dims/2] turns per position, factor on cos and sin) of a rotation's configuration."""
    dims, base = int(rot["dims"]), float(rot["base"])
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0
    factor, original = float(sc["factor"]), float(sc["original"])

    def place(turns):
        return dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo = max(math.floor(place(float(sc["fast"]))), 0)
    hi = min(math.ceil(place(float(sc["slow"]))), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / factor * ramp + fi * (1.0 - ramp))
    return out, 0.1 * math.log(factor) + 1.0


def turn(x, rot, pairs):
    """x [T, ..., n], row t at position t; `pairs` "neighbours" (2i with 2i+1) or "halves" (i with
    i + dims/2)."""
    f, mult = frequencies(rot)
    dims = int(rot["dims"])
    out = x.clone()
    p = torch.arange(x.shape[0], dtype=F64).view([-1] + [1] * (x.dim() - 2))
    for i, fi in enumerate(f):
        a, b = (2 * i, 2 * i + 1) if pairs == "neighbours" else (i, i + dims // 2)
        c, s = torch.cos(p * fi) * mult, torch.sin(p * fi) * mult
        u, v = x[..., a], x[..., b]
        out[..., a] = u * c - v * s
        out[..., b] = v * c + u * s
    return out


def softmax_with_sink(scores, sink):
    """scores [..., n]; sink: a number per leading entry (broadcastable) or None."""
    top = scores.max(-1, keepdim=True).values
    if sink is not None:
        top = torch.maximum(top, sink)
    e = torch.exp(scores - top)
    den = e.sum(-1, keepdim=True)
    if sink is not None:
        den = den + torch.exp(sink - top)
    return e / den


def latent_attention(h, w, m, kind, eps):
    """h [T, W] -> [T, W].  w: the layer's '.mix.*' tensors without the prefix."""
    T = h.shape[0]
    H, D, P, E, R = (int(m[k]) for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
    second = kind == "latent_attention_2"
    if second:
        q = rms_norm(h @ w["dq"].T, w["dq.norm"], eps) @ w["uq"].T
    else:
        q = h @ w["q"].T
    pairs = "halves" if second else "neighbours"
    q = q.view(T, H, D + P)
    down = h @ w["dkv"].T
    c = rms_norm(down[:, :R], w["dkv.norm"], eps)
    r = turn(down[:, R:], m["rot"], pairs)
    qr = turn(q[..., D:], m["rot"], pairs)
    k = (c @ w["uk"].T).view(T, H, D)
    v = (c @ w["uv"].T).view(T, H, E)
    s = torch.einsum("ihd,jhd->hij", q[..., :D], k) + torch.einsum("ihd,jd->hij", qr, r)
    s = s * float(m["scale"])
    s = s.masked_fill(torch.ones(T, T, dtype=torch.bool).triu(1), float("-inf"))
    p = softmax_with_sink(s, None if second else w["sink"].view(H, 1, 1))
    return torch.einsum("hij,jhe->ihe", p, v).reshape(T, H * E) @ w["o"].T


def dense_ff(h, w):
    return (gelu_tanh(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def capped_expert(h, gate_w, up_w, down_w, limit):
    g = torch.clamp(h @ gate_w.T, max=limit)
    u = torch.clamp(h @ up_w.T, -limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ down_w.T


def route(h, w, f):
    """[T, experts + identity] weights, zero where not chosen."""
    r = f["router"]
    top = int(r["top"])
    s = torch.softmax(h @ w["router"].T, -1)
    choice = s + w["correction"]
    out = torch.zeros_like(s)
    for t in range(h.shape[0]):
        order = sorted(range(s.shape[1]), key=lambda e: (-float(choice[t, e]), e))[:top]
        total = sum(s[t, e] for e in order) + 1e-20
        for e in order:
            out[t, e] = s[t, e] / total * float(r["scale"])
    return out


def routed_ff(h, w, f):
    """h [T, W]; w: the layer's '.mlp.*' tensors without the prefix; f: its configuration."""
    weights = route(h, w, f)
    n = int(f["router"]["experts"])
    out = weights[:, n:].sum(-1, keepdim=True) * h                     # identity experts
    for e in range(n):
        y = capped_expert(h, w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"], float(f["expert"]["limit"]))
        out = out + weights[:, e:e + 1] * y
    if f.get("shared"):
        out = out + capped_expert(h, w["shared.gate"], w["shared.up"], w["shared.down"],
                                  float(f["shared"]["limit"]))
    return out


def hyper_step(streams, sublayer, hc_in, hc_out, hc_mix, m):
    """streams: list of [T, W]; all new streams are formed from the old ones."""
    n = len(streams)
    y = sublayer(sum(hc_in[a] * streams[a] for a in range(n)))
    return [sum(hc_mix[a, b] * streams[a] for a in range(n)) + m * hc_out[b] * y for b in range(n)]


def forward(cfg, weights, tokens):
    """tokens: list of ids.  Returns (logits [T, vocab], [sum of the streams after every layer])."""
    w = {k: v.to(F64) for k, v in weights.items()}
    eps, m = float(cfg["norm"]["eps"]), float(cfg["residual_mult"])

    def norm(x, name):
        return tanh_norm(x, w[name + ".alpha"], w[name], w[name + ".b"])
    x = w["embed"][torch.tensor(tokens)] * float(cfg["embedding"]["scale"])
    streams = [x] * int(cfg["streams"])
    seen = []
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."

        def part(prefix):
            return {k[len(p + prefix):]: v for k, v in w.items() if k.startswith(p + prefix)}
        mixer, ff, f = part("mix."), part("mlp."), L.get("mlp")
        subs = [lambda u: latent_attention(norm(u, p + "norm1"), mixer, L["mixer"], L["type"], eps)]
        if f:
            subs.append(lambda u: (dense_ff(norm(u, p + "norm2"), ff) if f["kind"] == "dense"
                                   else routed_ff(norm(u, p + "norm2"), ff, f)))
        for q, sub in enumerate(subs, 1):
            streams = hyper_step(streams, sub, w[p + f"hc{q}.in"], w[p + f"hc{q}.out"],
                                 w[p + f"hc{q}.mix"], m)
        seen.append(sum(streams))
    return norm(sum(streams), "final.norm") @ w["head"].T, seen


def greedy(cfg, weights, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        logits, _ = forward(cfg, weights, toks)
        toks.append(int(torch.argmax(logits[-1])))
    return toks[len(prompt):]
