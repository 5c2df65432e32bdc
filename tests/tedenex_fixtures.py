"""Small Tedenex configurations and random checkpoints for the tests (made here, from the tensor
names and shapes the family's checkpoints use; nothing is read from outside)."""
from __future__ import annotations

import json
import os

import torch


def attention(heads=4, kv_heads=2, dim=10, vdim=12, conv=3, size=11, scale=0.3):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
                                           "conv": conv, "scale": scale, "mask": {"size": size}}}


def wkv(heads=3, dim=9):
    return {"type": "wkv", "mixer": {"heads": heads, "dim": dim}}


def latent(heads=4, dim=10, rot_dim=8, vdim=12, kv_rank=20, q_rank=14, scale=0.25, base=100.0):
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank,
                      "q_rank": q_rank, "scale": scale, "rot": {"base": base, "dims": rot_dim}}}


def dense(ff=28):
    return {"kind": "dense", "ff": ff}


def config(layers, width=40, vocab=89, eps=1e-5, side=6, loop=None):
    """``layers``: list of (mixer dict, mlp dict or None); ``loop``: (start, stop, times)."""
    c = {"architecture": "Tedenex", "vocab": vocab, "width": width, "norm": {"eps": eps},
         "token_side": {"dim": side}, "layers": [dict(m, mlp=f) for m, f in layers]}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


def default_config():
    """Every mixer with and without a feed-forward, a loop in the middle of the stack."""
    return config([(attention(), dense()), (wkv(), None), (latent(), dense(20)),
                   (attention(heads=3, kv_heads=3, dim=8, vdim=6, conv=4, size=16), None),
                   (wkv(heads=2, dim=16), dense(12))], loop=(1, 4, 2))


def mixer_shapes(kind, m, W, rank):
    H, D = m["heads"], m["dim"]
    if kind == "attention":
        G, E = m["kv_heads"], m["vdim"]
        out = [("q.norm", (D,)), ("k.norm", (D,)), ("o", (W, H * E))]
        for k, n in (("q", H * D), ("k", G * D), ("v", G * E)):
            out += [(k, (n, W)), (k + ".b", (n,)), (k + ".conv", (n, m["conv"]))]
        return out
    if kind == "wkv":
        return ([("mu." + k, (W,)) for k in "rkvgw"] + [(k, (H * D, W)) for k in "rkvg"]
                + [("w1", (rank, W)), ("w2", (H * D, rank)), ("w0", (H * D,)), ("u", (H, D)),
                   ("norm", (H * D,)), ("o", (W, H * D))])
    P, E, R, Q = (m[k] for k in ("rot_dim", "vdim", "kv_rank", "q_rank"))
    return [("dq", (Q, W)), ("dq.norm", (Q,)), ("uq", (H * (D + P), Q)), ("dkv", (R + P, W)),
            ("dkv.norm", (R,)), ("uk", (H * D, R)), ("uv", (H * E, R)), ("o", (W, H * E))]


def shapes(c, rank=5):
    W, V, n = c["width"], c["vocab"], c["token_side"]["dim"]
    yield "embed", (V, W)
    yield "side.embed", (V, n * len(c["layers"]))
    for i, L in enumerate(c["layers"]):
        p = f"l{i}."
        for nm in ("norm1", "norm1b") + (("norm2", "norm2b") if L["mlp"] else ()):
            yield p + nm, (W,)
        for nm, s in mixer_shapes(L["type"], L["mixer"], W, rank):
            yield p + "mix." + nm, s
        if L["mlp"]:
            yield p + "mlp.up", (L["mlp"]["ff"], W)
            yield p + "mlp.down", (W, L["mlp"]["ff"])
        yield p + "side.gate", (n, W)
        yield p + "side.proj", (W, n)
        yield p + "side.norm", (W,)
    yield "final.norm", (W,)


def weights(c, seed=0, rank=5):
    """Random tensors, rounded to bfloat16 (what a checkpoint holds).  Decays run from quick to
    slow, shifts and filters weigh past tokens about as much as the current one, biases are large
    enough that zeros ahead of a sequence differ from filtered biases."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in shapes(c, rank):
        leaf = name.rsplit(".", 1)[-1]
        r = torch.randn(shape, generator=g)
        if leaf in ("norm1", "norm1b", "norm2", "norm2b") or name == "final.norm":
            t = 0.2 * r
        elif leaf == "norm":
            t = 1.0 + 0.2 * r
        elif leaf == "conv":
            t = 0.6 * r
        elif leaf == "b":
            t = 0.5 * r
        elif ".mu." in name:
            t = 0.5 + 0.4 * r
        elif leaf == "w0":
            t = -2.0 + 1.5 * r
        elif leaf == "u" and ".mix." in name:
            t = r
        elif name in ("embed", "side.embed"):
            t = r
        else:
            t = r * shape[-1] ** -0.5
        out[name] = t.to(torch.bfloat16)
    return out


def save_checkpoint(folder, c, w):
    from safetensors.torch import save_file
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(c, f)
    save_file({k: v.contiguous() for k, v in w.items()}, os.path.join(folder, "model.safetensors"))
    return folder
