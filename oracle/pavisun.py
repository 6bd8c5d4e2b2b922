"""Plain PyTorch-CPU oracle of the Pavisun decoder (test infrastructure only, one function per mechanism).

Pavisun carries ``streams`` parallel residual streams (hyper-connections), all equal to the embedding row at first.  Sublayer q of a layer (1: mixer, 2: feed-forward)
reads u = sum_s a[s] x_s, computes y = sublayer(n(u)), n an RMS norm with a plain weight, and every stream becomes x_t <- sum_s M[s, t] x_s + b[t] y; the model's
output is the sum of the streams.  A run of neighbouring layers may be passed several times with the same weights, every pass with keys and values of its own.
Mixers:
  * *attention*   -- grouped-query softmax attention over a sliding window whose values are the unrotated keys; rotate-half rotary with frequencies and amplitude
    rescaled for a longer context (YaRN); capped scores;
  * *attention_2* -- grouped-query softmax attention over a sliding window that keeps the first tokens; no rotation, unit-RMS queries and keys, a per-head distance
    bias taken off the score, a sigmoid gate per output channel.
Feed-forward: SiLU-gated experts picked by a table of the token ids (no router), the mean of the picked experts.  A final norm, an untied head, capped logits.

Everything works on ONE whole sequence, in the dtype of the tensors handed in (fp32 or fp64), and shares no code with ``llm_quest_amd``.  ``weights`` maps the
checkpoint's tensor names to tensors; ``cfg`` is the parsed ``config.json``.
"""

import math

import torch


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def yarn(dims, base, scaling):
    """(frequencies as a list of floats, amplitude of cosine and sine)."""
    freqs = [float(base) ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not scaling:
        return freqs, 1.0
    factor, original = float(scaling["factor"]), float(scaling["original"])

    def dim_of(turns):
        return dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo, hi = max(math.floor(dim_of(scaling["fast"])), 0), min(math.ceil(dim_of(scaling["slow"])), dims - 1)
    out = []
    for i, f in enumerate(freqs):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / factor * ramp + f * (1.0 - ramp))
    return out, 0.1 * math.log(factor) + 1.0


def rotate_half(x, dims, freqs, amplitude):
    """x [T, H, D] at positions 0 .. T-1; entry i of the first ``dims`` turns with entry i + dims/2, the pair's length times ``amplitude``."""
    T, half = x.shape[0], dims // 2
    out = x.clone()
    pos = torch.arange(T, dtype=x.dtype)
    for i in range(half):
        ang = pos * torch.tensor(freqs[i], dtype=x.dtype)
        c, s = (torch.cos(ang) * amplitude)[:, None], (torch.sin(ang) * amplitude)[:, None]
        u, v = x[:, :, i], x[:, :, i + half]
        out[:, :, i] = u * c - v * s
        out[:, :, i + half] = v * c + u * s
    return out


def visible(T, size, keep_first=0):
    """[T, T] bool: row i sees column j."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    ok = j <= i
    if size:
        ok = ok & ((i - j < size) | (j < keep_first))
    return ok


def head_slope(h, heads):
    return 2.0 ** (-8.0 * (h + 1) / heads)


def softmax_head(q, k, v, scale, ok, softcap=0.0, slope=0.0):
    """One head over a whole sequence: q, k [T, d], v [T, dv], ok [T, T] the visible keys."""
    T = q.shape[0]
    s = (q @ k.T) * scale
    if softcap:
        s = softcap * torch.tanh(s / softcap)
    if slope:
        s = s - slope * (torch.arange(T)[:, None] - torch.arange(T)[None, :]).to(s.dtype)
    return torch.softmax(s.masked_fill(~ok, float("-inf")), dim=-1) @ v


def attention(h, w, p, m):
    T, H, G, d = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q, k = (h @ w[p + "q"].T).reshape(T, H, d), (h @ w[p + "k"].T).reshape(T, G, d)
    v = k
    rot = m.get("rot")
    if rot:
        freqs, amp = yarn(rot["dims"], rot["base"], rot.get("scaling"))
        q, k = rotate_half(q, rot["dims"], freqs, amp), rotate_half(k, rot["dims"], freqs, amp)
    ok = visible(T, m["mask"]["size"])
    o = [softmax_head(q[:, i], k[:, i // (H // G)], v[:, i // (H // G)], m["scale"], ok, m.get("softcap") or 0.0) for i in range(H)]
    return torch.cat(o, dim=1) @ w[p + "o"].T


def attention_2(h, w, p, m, eps):
    T, H, G, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k = unit_rms((h @ w[p + "q"].T).reshape(T, H, d), eps), unit_rms((h @ w[p + "k"].T).reshape(T, G, d), eps)
    v = (h @ w[p + "v"].T).reshape(T, G, dv)
    ok = visible(T, m["mask"]["size"], m["mask"].get("keep_first", 0))
    o = [softmax_head(q[:, i], k[:, i // (H // G)], v[:, i // (H // G)], m["scale"], ok, slope=head_slope(i, H)) for i in range(H)]
    return (torch.cat(o, dim=1) * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def expert(h, w, p):
    g = h @ w[p + "gate"].T
    return (g * torch.sigmoid(g) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def table_experts(h, tokens, w, p, mlp):
    top = mlp["router"]["top"]
    out = torch.zeros_like(h)
    for t, tok in enumerate(tokens):
        for e in w[p + "table"][int(tok)].tolist():
            out[t] += expert(h[t : t + 1], w, f"{p}e{e}.")[0] / top
    return out


def read_streams(xs, a):
    """xs [T, S, W], a [S] -> [T, W]."""
    return sum(a[s] * xs[:, s] for s in range(xs.shape[1]))


def write_streams(xs, y, mix, b):
    """Every stream t becomes sum_s mix[s, t] x_s + b[t] y."""
    S = xs.shape[1]
    return torch.stack([sum(mix[s, t] * xs[:, s] for s in range(S)) + b[t] * y for t in range(S)], dim=1)


def layer_runs(n_layers, loop):
    """The layers in the order they are run: start .. stop-1 ``times`` times, then the rest."""
    if not loop:
        return list(range(n_layers))
    return list(range(loop["start"])) + list(range(loop["start"], loop["stop"])) * loop["times"] + list(range(loop["stop"], n_layers))


def forward(cfg, weights, tokens, dtype=torch.float32, return_layers=False):
    """Logits [T, vocab] of one whole sequence (and the sum of the streams after every layer run)."""
    w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    xs = torch.stack([x] * cfg["streams"], dim=1)
    layers = []
    for i in layer_runs(len(cfg["layers"]), cfg.get("loop")):
        layer, p = cfg["layers"][i], f"l{i}."
        m = layer["mixer"]
        h = unit_rms(read_streams(xs, w[p + "hc1.in"]), eps) * w[p + "norm1"]
        y = attention(h, w, p + "mix.", m) if layer["type"] == "attention" else attention_2(h, w, p + "mix.", m, eps)
        xs = write_streams(xs, y, w[p + "hc1.mix"], w[p + "hc1.out"])
        if layer.get("mlp") is not None:
            h = unit_rms(read_streams(xs, w[p + "hc2.in"]), eps) * w[p + "norm2"]
            xs = write_streams(xs, table_experts(h, tokens, w, p + "mlp.", layer["mlp"]), w[p + "hc2.mix"], w[p + "hc2.out"])
        layers.append(xs.sum(1))
    logits = (unit_rms(xs.sum(1), eps) * w["final.norm"]) @ w["head"].T
    cap = cfg.get("logit_softcap")
    if cap:
        logits = cap * torch.tanh(logits / cap)
    return (logits, layers) if return_layers else logits
