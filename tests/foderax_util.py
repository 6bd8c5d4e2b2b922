"""Small random Foderax checkpoints for the tests: a config dict and a name -> tensor dict in the checkpoint's naming, optionally written to a folder
(config.json + model.safetensors) so the tests go through the registry and the loader like a user does."""

import json
import os

import torch


def latent(heads=3, dim=20, vdim=28, q_rank=36, kv_rank=44, scale=None):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": dim ** -0.5 if scale is None else scale}}


def diff(heads=4, kv_heads=2, dim=16, vdim=24, rot_dims=12, base=5000.0, scale=None, diff=0.4, kv_from=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": dim ** -0.5 if scale is None else scale, "diff": diff, "rot": {"dims": rot_dims, "base": base}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m}


def parallel(heads=6, kv_heads=2, dim=24, vdim=20, rot_dims=16, base=300.0, scale=None, width=52, left_scale=0.7, right_scale=1.3):
    return {"type": "parallel", "mixer": {"left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": dim ** -0.5 if scale is None else scale,
                                                   "rot": {"dims": rot_dims, "base": base}},
                                          "right": {"width": width}, "left_scale": left_scale, "right_scale": right_scale}}


def moe(experts=6, top=2, ff=40, count=3, keep=2):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, "groups": {"count": count, "keep": keep}}}


def make_config(layers, width=72, vocab=131, eps=1e-5, scale=3.0, softcap=9.0):
    """layers: list of (mixer entry, mlp entry or None)."""
    return {"architecture": "Foderax", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale}, "logit_softcap": softcap,
            "layers": [dict(mixer, mlp=mlp) for mixer, mlp in layers]}


def make_weights(cfg, seed=0):
    g = torch.Generator().manual_seed(seed)
    W = cfg["width"]
    bf = torch.bfloat16

    def lin(o, i, gain=1.0):
        return (torch.randn(o, i, generator=g) * gain / i ** 0.5).to(bf)

    def vec(n, mean=1.0, std=0.1):
        return (mean + std * torch.randn(n, generator=g)).to(bf)

    w = {"embed": lin(cfg["vocab"], W, 2.0), "final.norm": vec(W, 0.0, 0.2)}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        w[p + "norm1"], w[p + "ls1"], w[p + "dwa"] = vec(W, 0.0, 0.2), vec(W, 0.8, 0.3), vec(i + 2, 0.3, 0.4)
        x = p + "mix."
        if layer["type"] == "latent_attention":
            H, d, dv, rq, r = m["heads"], m["dim"], m["vdim"], m["q_rank"], m["kv_rank"]
            w[x + "dq"], w[x + "dq.norm"], w[x + "uq"] = lin(rq, W), vec(rq), lin(H * d, rq, 3.0)
            w[x + "dkv"], w[x + "dkv.norm"], w[x + "uk"], w[x + "uv"] = lin(r, W), vec(r), lin(H * d, r, 2.0), lin(H * dv, r)
            w[x + "sink"], w[x + "g"], w[x + "o"] = vec(H, 1.5, 1.0), lin(H, W, 2.0), lin(W, H * dv)
        elif layer["type"] == "attention":
            H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            w[x + "q"], w[x + "q.b"] = lin(2 * H * d, W, 3.0), vec(2 * H * d, 0.0, 0.3)
            if m.get("kv_from") is None:
                w[x + "k"], w[x + "k.b"], w[x + "v"], w[x + "v.b"] = lin(2 * G * d, W, 2.0), vec(2 * G * d, 0.0, 0.3), lin(G * dv, W), vec(G * dv, 0.0, 0.3)
            for s in ("lq1", "lk1", "lq2", "lk2"):
                w[x + s] = vec(d, 0.0, 1.0 / d ** 0.25)
            w[x + "g"], w[x + "o"] = lin(H * dv, W, 1.5), lin(W, H * dv)
        else:
            L, C = m["left"], m["right"]["width"]
            H, G, d, dv = L["heads"], L["kv_heads"], L["dim"], L["vdim"]
            l, r = x + "left.", x + "right."
            w[l + "q"], w[l + "k"], w[l + "v"], w[l + "pb"], w[l + "o"] = lin(H * d, W, 3.0), lin(G * d, W, 2.0), lin(G * dv, W), vec(H, -3.0, 1.0), lin(W, H * dv)
            w[r + "z"], w[r + "z.b"], w[r + "x"], w[r + "x.b"] = lin(C, W, 2.0), vec(C, -1.0, 1.0), lin(C, W), vec(C, 0.0, 0.3)
            w[r + "g"], w[r + "o"] = lin(C, W), lin(W, C)
        mlp = layer.get("mlp")
        if mlp:
            w[p + "ls2"] = vec(W, 0.8, 0.3)
            e, E, F = p + "mlp.", mlp["router"]["experts"], mlp["expert"]["ff"]
            w[e + "router"] = lin(E, W, 2.0)
            for j in range(E):
                w[f"{e}e{j}.up"], w[f"{e}e{j}.down"] = lin(F, W, 1.5), lin(W, F)
    return w


def save(folder, cfg, weights):
    from safetensors.torch import save_file

    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in weights.items()}, os.path.join(folder, "model.safetensors"))
    return folder


def default_layers():
    """Every mixer; a layer without feed-forward; two layers on one layer's keys and values (one of them not its neighbour); head groups of 2, 3 and 1."""
    return [(parallel(), moe()),
            (diff(), None),
            (latent(), moe(experts=8, top=3, ff=24, count=4, keep=2)),
            (diff(kv_from=1, diff=0.7, scale=0.3), moe()),
            (diff(heads=3, kv_heads=1, dim=10, vdim=32, rot_dims=10, base=40.0), moe(experts=5, top=1, ff=33, count=1, keep=1)),
            (parallel(heads=4, kv_heads=4, dim=8, vdim=12, rot_dims=8, width=40, left_scale=1.2, right_scale=0.4), None),
            (diff(heads=6, kv_heads=2, kv_from=1, diff=0.2), moe(experts=6, top=2, ff=20, count=6, keep=3))]
