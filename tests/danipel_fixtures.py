"""Small Danipel configurations and random checkpoints for the tests (made here, from the tensor
names and shapes the family's checkpoints use; nothing is read from outside)."""
from __future__ import annotations

import json
import os

import torch

YARN = {"factor": 4.0, "original": 64, "fast": 8.0, "slow": 1.0}


def latent(kind=1, heads=4, dim=10, rot_dim=8, vdim=12, kv_rank=20, q_rank=14, scale=0.25, base=100.0,
           scaling=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale,
         "rot": {"base": base, "dims": rot_dim}}
    if scaling:
        m["rot"]["scaling"] = dict(scaling)
    if kind == 2:
        m["q_rank"] = q_rank
    return {"type": "latent_attention" if kind == 1 else "latent_attention_2", "mixer": m}


def dense(ff=28):
    return {"kind": "dense", "ff": ff}


def moe(experts=5, identity=2, top=3, ff=12, limit=1.5, scale=1.7, shared_ff=20, shared_limit=0.8):
    f = {"kind": "moe", "expert": {"ff": ff, "limit": limit},
         "router": {"experts": experts, "identity": identity, "scale": scale, "top": top}}
    if shared_ff:
        f["shared"] = {"ff": shared_ff, "limit": shared_limit}
    return f


def config(layers, width=40, vocab=89, eps=1e-5, streams=3, residual_mult=0.6, embed_scale=3.0):
    """``layers``: list of (mixer dict, mlp dict or None)."""
    return {"architecture": "Danipel", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "embedding": {"scale": embed_scale}, "residual_mult": residual_mult, "streams": streams,
            "layers": [dict(m, mlp=f) for m, f in layers]}


def default_config():
    """Both mixers, both kinds of feed-forward, a layer without one, experts without a shared one
    and without identity experts."""
    return config([(latent(2), dense()), (latent(1, scaling=YARN), moe()),
                   (latent(1, heads=3, dim=6, rot_dim=4, vdim=5, kv_rank=16, base=1000.0), None),
                   (latent(2, heads=2, dim=16, rot_dim=6, vdim=8, kv_rank=12, q_rank=20),
                    moe(experts=4, identity=0, top=2, ff=8, scale=1.0, shared_ff=0))])


def mixer_shapes(kind, m, W):
    H, D, P, E, R = (m[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
    out = [("dkv", (R + P, W)), ("dkv.norm", (R,)), ("uk", (H * D, R)), ("uv", (H * E, R)), ("o", (W, H * E))]
    if kind == "latent_attention_2":
        Q = m["q_rank"]
        return [("dq", (Q, W)), ("dq.norm", (Q,)), ("uq", (H * (D + P), Q))] + out
    return [("q", (H * (D + P), W)), ("sink", (H,))] + out


def ff_shapes(f, W):
    if f["kind"] == "dense":
        n = f["ff"]
        return [("gate", (n, W)), ("up", (n, W)), ("down", (W, n))]
    names = [(f"e{e}.", f["expert"]["ff"]) for e in range(f["router"]["experts"])]
    if f.get("shared"):
        names.append(("shared.", f["shared"]["ff"]))
    out = []
    for n, s in names:
        out += [(n + "gate", (s, W)), (n + "up", (s, W)), (n + "down", (W, s))]
    rows = f["router"]["experts"] + f["router"]["identity"]
    return out + [("router", (rows, W)), ("correction", (rows,))]


def shapes(c):
    W, V, S = c["width"], c["vocab"], c["streams"]
    yield "embed", (V, W)
    yield "head", (V, W)
    for i, L in enumerate(c["layers"]):
        parts = [("mix.", mixer_shapes(L["type"], L["mixer"], W))]
        if L["mlp"]:
            parts.append(("mlp.", ff_shapes(L["mlp"], W)))
        for q, (prefix, names) in enumerate(parts, 1):
            p = f"l{i}."
            for n, s in ((f"norm{q}", (W,)), (f"norm{q}.b", (W,)), (f"norm{q}.alpha", ()), (f"hc{q}.in", (S,)),
                         (f"hc{q}.out", (S,)), (f"hc{q}.mix", (S, S))):
                yield p + n, s
            for n, s in names:
                yield p + prefix + n, s
    for n, s in (("final.norm", (W,)), ("final.norm.b", (W,)), ("final.norm.alpha", ())):
        yield n, s


def weights(c, seed=0, qk_gain=2.0):
    """Random tensors, rounded to bfloat16 (what a checkpoint holds); queries and keys are scaled
    up so that softmaxes are peaked, router rows so that the choice is rarely a close call, the
    experts' inputs so that the clamps bite; the streams' mix is far from symmetric."""
    g = torch.Generator().manual_seed(seed)
    S = c["streams"]
    out = {}
    for name, shape in shapes(c):
        leaf = name.rsplit(".", 1)[-1]
        r = torch.randn(shape, generator=g)
        if leaf in ("norm", "norm1", "norm2"):
            t = 1.0 + 0.2 * r
        elif leaf == "alpha":
            t = 0.6 + 0.1 * r
        elif leaf == "b":
            t = 0.2 * r
        elif leaf == "in":
            t = (1.0 + 0.4 * r) / S
        elif leaf == "out":
            t = 1.0 + 0.3 * r
        elif leaf == "mix":
            t = torch.eye(S) * 0.8 + 0.2 * r
        elif leaf == "sink":
            t = 1.5 * r
        elif leaf == "correction":
            t = 0.15 * r
        elif name == "embed":
            t = r / c["embedding"]["scale"]
        else:
            gain = qk_gain if leaf in ("q", "uq", "router", "gate", "up") else 1.0
            t = r * shape[-1] ** -0.5 * gain
        out[name] = t.to(torch.bfloat16)
    return out


def save_checkpoint(folder, c, w):
    from safetensors.torch import save_file
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(c, f)
    save_file({k: v.contiguous() for k, v in w.items()}, os.path.join(folder, "model.safetensors"))
    return folder
