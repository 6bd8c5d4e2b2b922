"""Small random Pavisun checkpoints for the tests: a config dict and a name -> tensor dict in the checkpoint's naming, optionally written to a folder
(config.json + model.safetensors) so the tests go through the registry and the loader like a user does."""

import json
import os

import torch


def attention(heads=4, kv_heads=2, dim=24, size=13, rot_dims=16, base=2000.0, scaling=(4.0, 64, 8.0, 1.0), scale=None, softcap=6.0):
    """``scaling``: (factor, original, fast, slow) or None."""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "mask": {"size": size}, "scale": dim ** -0.5 if scale is None else scale}
    if rot_dims:
        m["rot"] = {"dims": rot_dims, "base": base}
        if scaling:
            m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    if softcap:
        m["softcap"] = softcap
    return {"type": "attention", "mixer": m}


def attention_2(heads=6, kv_heads=2, dim=16, vdim=40, size=11, keep_first=5, scale=0.5):
    return {"type": "attention_2", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": size, "keep_first": keep_first}, "scale": scale}}


def moe(experts=7, top=2, ff=40):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def make_config(layers, width=72, vocab=131, eps=1e-5, streams=4, softcap=20.0, loop=None):
    """layers: list of (mixer entry, mlp entry or None); loop: (start, stop, times)."""
    cfg = {"architecture": "Pavisun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "streams": streams, "layers": [dict(mixer, mlp=mlp) for mixer, mlp in layers]}
    if softcap:
        cfg["logit_softcap"] = softcap
    if loop:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


def make_weights(cfg, seed=0):
    g = torch.Generator().manual_seed(seed)
    W, n = cfg["width"], cfg["streams"]
    bf = torch.bfloat16

    def lin(o, i, gain=1.0):
        return (torch.randn(o, i, generator=g) * gain / i ** 0.5).to(bf)

    def vec(k, mean=1.0, std=0.2):
        return (mean + std * torch.randn(k, generator=g)).to(bf)

    w = {"embed": (2.0 * torch.randn(cfg["vocab"], W, generator=g)).to(bf), "head": lin(cfg["vocab"], W, 3.0), "final.norm": vec(W)}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        x = p + "mix."
        w[x + "q"], w[x + "k"], w[x + "o"] = lin(H * d, W, 1.5), lin(G * d, W), lin(W, H * dv)
        if layer["type"] == "attention_2":
            w[x + "v"], w[x + "g"] = lin(G * dv, W), lin(H * dv, W, 1.5)
        mlp = layer.get("mlp")
        for q in (1, 2) if mlp else (1,):
            w[f"{p}norm{q}"] = vec(W)
            w[f"{p}hc{q}.in"], w[f"{p}hc{q}.out"] = vec(n, 1.0, 0.3), vec(n, 0.5, 0.4)
            w[f"{p}hc{q}.mix"] = (0.8 * torch.eye(n) + 0.2 * torch.randn(n, n, generator=g) / n ** 0.5).to(bf)
        if mlp:
            e, E, F, top = p + "mlp.", mlp["router"]["experts"], mlp["expert"]["ff"], mlp["router"]["top"]
            w[e + "table"] = torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(cfg["vocab"])]).to(torch.int32)
            for j in range(E):
                w[f"{e}e{j}.gate"], w[f"{e}e{j}.up"], w[f"{e}e{j}.down"] = lin(F, W, 1.2), lin(F, W), lin(W, F)
    return w


def save(folder, cfg, weights):
    from safetensors.torch import save_file

    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in weights.items()}, os.path.join(folder, "model.safetensors"))
    return folder


def default_layers():
    """Both mixers; a layer without feed-forward; head groups of 1, 2 and 3; a window smaller than, equal to and larger than what it keeps."""
    return [(attention(), moe()),
            (attention_2(), moe(experts=5, top=3, ff=24)),
            (attention(heads=3, kv_heads=3, dim=10, size=30, rot_dims=10, base=40.0, scaling=None, softcap=0.0), None),
            (attention_2(heads=4, kv_heads=4, dim=12, vdim=8, size=4, keep_first=9, scale=0.3), moe(experts=6, top=1, ff=33)),
            (attention(heads=6, kv_heads=2, dim=32, size=7, rot_dims=20, base=500.0, scaling=(16.0, 40, 4.0, 0.5)), moe(experts=4, top=4, ff=20))]
