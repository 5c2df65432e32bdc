"""Plain float64 restatement of the Tedenex decoder, one function per mechanism.  It shares no code
with the package: the tests compare the engine with it.

The design in this file's notation (W = width, eps = the norms' epsilon, everywhere inside the root):

* x = E[token]; the table E is also the output projection, behind the final norm;
* norm(x) = x / rms(x) (1 + w) around every sublayer: x <- x + norm_b(f(norm_a(x))) for a mixer,
  then for a feed-forward, which may be absent;
* behind both, a per-layer token input: with e the layer's run of `dim` numbers of a second table's
  row, x <- x + n(P (gelu_tanh(G x) e)), n(y) = y / rms(y) w;
* layers start .. stop - 1 run `times` times; ahead of every pass but the first E[token] is added;
* mixer "attention": biased q, k, v; a causal filter over time on every projected channel; each q
  and k head / rms, times a weight the heads share; score = scale (q . k) - 2^(-8 (h+1) / H) (i - j)
  over the keys j <= i of the query's own chunk of `size` positions; softmax;
* mixer "wkv": with d = h_(t-1) - h_t (h_(-1) = 0), the inputs of r, k, v, gate and decay are
  h + mu d; w = exp(-exp(W2 tanh(W1 .) + w0)); per head o = (S + diag(u) k v^T)^T r, then
  S <- diag(w) S + k v^T; o / rms(o) per head, times a weight, times silu(gate);
* mixer "latent_attention": c = rmsnorm of the first R rows of W_dkv h, rot = the last P rows,
  turned; head h's key is [W_uk_h c | rot], its value W_uv_h c; q = W_uq rmsnorm(W_dq h) per head =
  [D unrotated | P turned]; pairs of neighbours turn; score = scale (q . k); all j <= i; softmax;
* feed-forward: W_down relu(W_up h)^2.
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def time_filter(u, w):
    """u [T, C], w [C, taps]: y_t = sum_j w[:, j] u_(t - taps + 1 + j), zeros before the start."""
    taps = w.shape[1]
    y = torch.zeros_like(u)
    for j in range(taps):
        back = taps - 1 - j
        y[back:] += w[:, j] * u[:max(u.shape[0] - back, 0)]
    return y


def attention(h, w, m, eps):
    """h [T, W] -> [T, W].  w: the layer's '.mix.*' tensors without the prefix."""
    T = h.shape[0]
    H, G, D, E = (int(m[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
    size = int(m["mask"]["size"])
    q, k, v = (time_filter(h @ w[n].T + w[n + ".b"], w[n + ".conv"]) for n in "qkv")
    q = unit_rms(q.view(T, H, D), eps) * w["q.norm"]
    k = unit_rms(k.view(T, G, D), eps) * w["k.norm"]
    v = v.view(T, G, E)
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    hidden = (j > i) | (torch.div(i, size, rounding_mode="floor") != torch.div(j, size, rounding_mode="floor"))
    out = torch.zeros(T, H, E, dtype=F64)
    for hd in range(H):
        g = hd // (H // G)
        s = q[:, hd] @ k[:, g].T * float(m["scale"]) - 2.0 ** (-8.0 * (hd + 1) / H) * (i - j)
        out[:, hd] = torch.softmax(s.masked_fill(hidden, float("-inf")), -1) @ v[:, g]
    return out.reshape(T, H * E) @ w["o"].T


def wkv(h, w, m, eps):
    T = h.shape[0]
    H, D = int(m["heads"]), int(m["dim"])
    prev = torch.cat([torch.zeros_like(h[:1]), h[:-1]], 0)

    def mixed(n):
        return h + (prev - h) * w["mu." + n]
    r, k, v = ((mixed(n) @ w[n].T).view(T, H, D) for n in "rkv")
    gate = mixed("g") @ w["g"].T
    gate = gate * torch.sigmoid(gate)
    decay = torch.exp(-torch.exp(torch.tanh(mixed("w") @ w["w1"].T) @ w["w2"].T + w["w0"])).view(T, H, D)
    o = torch.zeros(T, H, D, dtype=F64)
    for hd in range(H):
        S = torch.zeros(D, D, dtype=F64)
        for t in range(T):
            kv = torch.outer(k[t, hd], v[t, hd])
            o[t, hd] = (S + w["u"][hd][:, None] * kv).T @ r[t, hd]
            S = decay[t, hd][:, None] * S + kv
    o = unit_rms(o, eps).reshape(T, H * D) * w["norm"] * gate
    return o @ w["o"].T


def turn(x, base, dims):
    """x [T, ..., n], row t at position t: entries 2i and 2i + 1 (i < dims/2) turn by t base^(-2i/dims)."""
    out = x.clone()
    p = torch.arange(x.shape[0], dtype=F64).view([-1] + [1] * (x.dim() - 2))
    for i in range(dims // 2):
        a = p * base ** (-2.0 * i / dims)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * torch.cos(a) - v * torch.sin(a)
        out[..., 2 * i + 1] = v * torch.cos(a) + u * torch.sin(a)
    return out


def latent_attention(h, w, m, eps):
    T = h.shape[0]
    H, D, P, E, R = (int(m[k]) for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
    base, dims = float(m["rot"]["base"]), int(m["rot"]["dims"])
    q = ((unit_rms(h @ w["dq"].T, eps) * w["dq.norm"]) @ w["uq"].T).view(T, H, D + P)
    down = h @ w["dkv"].T
    c = unit_rms(down[:, :R], eps) * w["dkv.norm"]
    rot, q_rot = turn(down[:, R:], base, dims), turn(q[..., D:], base, dims)
    k, v = (c @ w["uk"].T).view(T, H, D), (c @ w["uv"].T).view(T, H, E)
    s = torch.einsum("ihd,jhd->hij", q[..., :D], k) + torch.einsum("ihd,jd->hij", q_rot, rot)
    s = (s * float(m["scale"])).masked_fill(torch.ones(T, T, dtype=torch.bool).triu(1), float("-inf"))
    return torch.einsum("hij,jhe->ihe", torch.softmax(s, -1), v).reshape(T, H * E) @ w["o"].T


MIXERS = {"attention": attention, "wkv": wkv, "latent_attention": latent_attention}


def dense_ff(h, w):
    return torch.clamp(h @ w["up"].T, min=0.0) ** 2 @ w["down"].T


def token_input(x, e, w, eps):
    """What a layer's token input adds to x [T, W]; e [T, dim]: the layer's part of the token rows."""
    y = (gelu_tanh(x @ w["gate"].T) * e) @ w["proj"].T
    return unit_rms(y, eps) * w["norm"]


def run_order(cfg):
    """[(layer, its pass adds the embedding ahead of it)] in the order the layers run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    out = [(i, False) for i in range(a)]
    for p in range(loop["times"]):
        out += [(i, p > 0 and i == a) for i in range(a, b)]
    return out + [(i, False) for i in range(b, n)]


def forward(cfg, weights, tokens):
    """tokens: list of ids.  Returns (logits [T, vocab], [x after every layer run])."""
    w = {k: v.to(F64) for k, v in weights.items()}
    eps, dim = float(cfg["norm"]["eps"]), int(cfg["token_side"]["dim"])
    ids = torch.tensor(tokens)

    def norm(x, name):
        return unit_rms(x, eps) * (1.0 + w[name])
    x0 = w["embed"][ids]
    x, seen = x0, []
    for i, again in run_order(cfg):
        L, p = cfg["layers"][i], f"l{i}."

        def part(prefix):
            return {k[len(p + prefix):]: v for k, v in w.items() if k.startswith(p + prefix)}
        if again:
            x = x + x0
        x = x + norm(MIXERS[L["type"]](norm(x, p + "norm1"), part("mix."), L["mixer"], eps), p + "norm1b")
        if L.get("mlp"):
            x = x + norm(dense_ff(norm(x, p + "norm2"), part("mlp.")), p + "norm2b")
        x = x + token_input(x, w["side.embed"][ids][:, i * dim:(i + 1) * dim], part("side."), eps)
        seen.append(x)
    return norm(x, "final.norm") @ w["embed"].T, seen


def greedy(cfg, weights, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        logits, _ = forward(cfg, weights, toks)
        toks.append(int(torch.argmax(logits[-1])))
    return toks[len(prompt):]
