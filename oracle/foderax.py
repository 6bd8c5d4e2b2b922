"""Plain PyTorch-CPU oracle of the Foderax decoder (test infrastructure only, one function per mechanism).

Foderax is a pre-norm decoder with PARALLEL sublayers and a depth average.  With X_0 the embedding output and x_0 = X_0, layer i computes
    h = n(x_i),   X_(i+1) = x_i + s1 * mixer(h) + s2 * ff(h),   x_(i+1) = sum_(j <= i+1) d_i[j] X_j,
n an RMS norm whose weight is stored around zero (times 1 + w), s1 / s2 per-channel layer scales, d_i the layer's i + 2 depth weights.  Mixers:
  * *attention*        -- differential attention: two softmax maps per head over the same values, o = a1 - lambda a2, unit RMS per head times 1 - diff, a
    sigmoid gate per channel; a layer may read another layer's keys and values;
  * *latent_attention* -- keys and values from one normalised latent, no positions, a learned sink per head in the denominator, one sigmoid gate per head;
  * *parallel*         -- sigmoid attention (the weight of a key is sigmoid(score + bias_h), no softmax) beside a minimal gated recurrence whose gates read the
    current token only; a weighted sum of the two.
Feed-forward: softmax-scored experts chosen inside the best groups (a group's score is its largest), squared-ReLU, weights not renormalised.  The logits
come from the embedding table and pass cap * tanh(logits / cap).

Everything works on ONE whole sequence, in the dtype of the tensors handed in (fp32 or fp64), token by token where a recurrence is involved, and shares no
code with ``llm_quest_amd``.  ``weights`` maps the checkpoint's tensor names to tensors; ``cfg`` is the parsed ``config.json``.
"""

import torch


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def centred_rms(x, w, eps):
    """RMS norm, the weight stored around zero."""
    return unit_rms(x, eps) * (1.0 + w)


def rotate(x, dims, base, interleaved):
    """x [T, H, D] at positions 0 .. T-1; the first ``dims`` entries turn: neighbours (2i, 2i+1), or entry i with entry i + dims/2."""
    T = x.shape[0]
    out = x.clone()
    for i in range(dims // 2):
        a, b = (2 * i, 2 * i + 1) if interleaved else (i, i + dims // 2)
        f = float(base) ** (-2.0 * i / dims)
        pos = torch.arange(T, dtype=torch.float64)
        ang = pos * f if x.dtype == torch.float64 else pos.float() * torch.tensor(f, dtype=torch.float32)
        c, s = torch.cos(ang)[:, None].to(x.dtype), torch.sin(ang)[:, None].to(x.dtype)
        u, v = x[:, :, a], x[:, :, b]
        out[:, :, a] = u * c - v * s
        out[:, :, b] = v * c + u * s
    return out


def softmax_map(q, k, v, scale, sink=None):
    """One head over a whole sequence: q, k [T, d], v [T, dv]; row i sees j <= i; ``sink``: exp(sink) joins the denominator."""
    T = q.shape[0]
    s = (q @ k.T) * scale
    s = s.masked_fill(torch.ones(T, T, dtype=torch.bool).triu(1), float("-inf"))
    m = s.max(dim=1, keepdim=True).values
    if sink is not None:
        m = torch.maximum(m, sink)
    e = torch.exp(s - m)
    den = e.sum(dim=1, keepdim=True)
    if sink is not None:
        den = den + torch.exp(sink - m)
    return (e / den) @ v


def sigmoid_map(q, k, v, scale, bias):
    """One head without a softmax: the weight of a visible key is sigmoid(score + bias)."""
    T = q.shape[0]
    wt = torch.sigmoid((q @ k.T) * scale + bias)
    return wt.masked_fill(torch.ones(T, T, dtype=torch.bool).triu(1), 0.0) @ v


def diff_lambda(w, p, diff):
    return torch.exp((w[p + "lq1"] * w[p + "lk1"]).sum()) - torch.exp((w[p + "lq2"] * w[p + "lk2"]).sum()) + diff


def differential_kv(h, w, p, m):
    """The layer's keys [T, G, 2, dim] (rotated) and values [T, G, vdim]."""
    T, G, d = h.shape[0], m["kv_heads"], m["dim"]
    k = (h @ w[p + "k"].T + w[p + "k.b"]).reshape(T, 2 * G, d)
    v = (h @ w[p + "v"].T + w[p + "v.b"]).reshape(T, G, m["vdim"])
    rot = m.get("rot")
    if rot:
        k = rotate(k, rot["dims"], rot["base"], True)
    return k.reshape(T, G, 2, d), v


def differential_attention(h, w, p, m, eps, kv):
    T, H, G, d = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    k, v = kv
    q = (h @ w[p + "q"].T + w[p + "q.b"]).reshape(T, 2 * H, d)
    rot = m.get("rot")
    if rot:
        q = rotate(q, rot["dims"], rot["base"], True)
    q = q.reshape(T, H, 2, d)
    lam = diff_lambda(w, p, m["diff"])
    outs = []
    for hd in range(H):
        g = hd // (H // G)
        a1, a2 = (softmax_map(q[:, hd, mp], k[:, g, mp], v[:, g], m["scale"]) for mp in (0, 1))
        outs.append(unit_rms(a1 - lam * a2, eps) * (1.0 - m["diff"]))
    o = torch.cat(outs, dim=1) * torch.sigmoid(h @ w[p + "g"].T)
    return o @ w[p + "o"].T


def latent_attention(h, w, p, m, eps):
    T, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    cq = unit_rms(h @ w[p + "dq"].T, eps) * w[p + "dq.norm"]
    c = unit_rms(h @ w[p + "dkv"].T, eps) * w[p + "dkv.norm"]
    q = (cq @ w[p + "uq"].T).reshape(T, H, d)
    k = (c @ w[p + "uk"].T).reshape(T, H, d)
    v = (c @ w[p + "uv"].T).reshape(T, H, dv)
    gate = torch.sigmoid(h @ w[p + "g"].T)
    o = [softmax_map(q[:, hd], k[:, hd], v[:, hd], m["scale"], w[p + "sink"][hd]) * gate[:, hd : hd + 1] for hd in range(H)]
    return torch.cat(o, dim=1) @ w[p + "o"].T


def sigmoid_attention(h, w, p, m):
    T, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    G = m["kv_heads"]
    q, k, v = (h @ w[p + "q"].T).reshape(T, H, d), (h @ w[p + "k"].T).reshape(T, G, d), (h @ w[p + "v"].T).reshape(T, G, dv)
    rot = m.get("rot")
    if rot:
        q, k = (rotate(t, rot["dims"], rot["base"], False) for t in (q, k))
    o = [sigmoid_map(q[:, hd], k[:, hd // (H // G)], v[:, hd // (H // G)], m["scale"], w[p + "pb"][hd]) for hd in range(H)]
    return torch.cat(o, dim=1) @ w[p + "o"].T


def candidate(u):
    return torch.where(u >= 0, u + 0.5, torch.sigmoid(u))


def min_gru_states(zr, u):
    """zr, u [T, C] (gate logits and candidate inputs) -> the states [T, C], from zero."""
    z = torch.sigmoid(zr)
    S = torch.zeros(u.shape[1], dtype=u.dtype)
    out = []
    for t in range(u.shape[0]):
        S = (1.0 - z[t]) * S + z[t] * candidate(u[t])
        out.append(S)
    return torch.stack(out)


def min_gru(h, w, p):
    S = min_gru_states(h @ w[p + "z"].T + w[p + "z.b"], h @ w[p + "x"].T + w[p + "x.b"])
    g = h @ w[p + "g"].T
    return (S * g * torch.sigmoid(g)) @ w[p + "o"].T


def parallel_mixer(h, w, p, m):
    return m["left_scale"] * sigmoid_attention(h, w, p + "left.", m["left"]) + m["right_scale"] * min_gru(h, w, p + "right.")


def route(logits, router):
    """(ids [T, top], weights [T, top], gap [T]): softmax over all experts; only experts of the ``keep`` groups with the largest members are eligible; the
    ``top`` largest win with their own scores.  ``gap``: how close (in log score) the choice of groups or of experts was."""
    T, E = logits.shape
    s = torch.softmax(logits, dim=-1)
    top, gr = router["top"], router.get("groups") or {"count": 1, "keep": 1}
    n, keep = gr["count"], gr["keep"]
    ids, wts, gaps = [], [], []
    for t in range(T):
        best = s[t].reshape(n, E // n).max(dim=1).values
        order = torch.argsort(best, descending=True)
        gap = float("inf")
        if keep < n:
            gap = float(torch.log(best[order[keep - 1]]) - torch.log(best[order[keep]]))
        ok = torch.zeros(n, dtype=torch.bool)
        ok[order[:keep]] = True
        el = torch.where(ok.repeat_interleave(E // n), s[t], torch.full_like(s[t], -1.0))
        o = torch.argsort(el, descending=True)
        if top < keep * (E // n):
            gap = min(gap, float(torch.log(el[o[top - 1]]) - torch.log(el[o[top]])))
        ids.append(o[:top])
        wts.append(s[t][o[:top]])
        gaps.append(gap)
    return torch.stack(ids), torch.stack(wts), torch.tensor(gaps)


def expert(h, w, p):
    return torch.relu(h @ w[p + "up"].T) ** 2 @ w[p + "down"].T


def moe_ff(h, w, p, mlp, gaps=None):
    ids, wts, gap = route(h @ w[p + "router"].T, mlp["router"])
    if gaps is not None:
        gaps.append(gap)
    out = torch.zeros(h.shape[0], w[p + "e0.down"].shape[0], dtype=h.dtype)
    for e in range(mlp["router"]["experts"]):
        rows, slot = (ids == e).nonzero(as_tuple=True)
        if len(rows):
            out[rows] += wts[rows, slot][:, None] * expert(h[rows], w, f"{p}e{e}.")
    return out


def forward(cfg, weights, tokens, dtype=torch.float32, return_layers=False, gaps=None):
    """Logits [T, vocab] of one whole sequence (and the averaged residual stream after every layer).  ``gaps`` (a list) collects, per routed layer, every
    token's router gap (``route``)."""
    w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)] * float((cfg.get("embedding") or {}).get("scale", 1.0))
    results, layers, kvs = [x], [], {}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        h = centred_rms(x, w[p + "norm1"], eps)
        if layer["type"] == "attention":
            j = m.get("kv_from")
            kvs[i] = differential_kv(h, w, p + "mix.", m) if j is None else kvs[j]
            y = differential_attention(h, w, p + "mix.", m, eps, kvs[i])
        elif layer["type"] == "latent_attention":
            y = latent_attention(h, w, p + "mix.", m, eps)
        else:
            y = parallel_mixer(h, w, p + "mix.", m)
        new = x + w[p + "ls1"] * y
        if layer.get("mlp") is not None:
            new = new + w[p + "ls2"] * moe_ff(h, w, p + "mlp.", layer["mlp"], gaps)
        results.append(new)
        x = sum(w[p + "dwa"][j] * results[j] for j in range(i + 2))
        layers.append(x)
    logits = centred_rms(x, w["final.norm"], eps) @ w["embed"].T
    cap = cfg.get("logit_softcap")
    if cap:
        logits = cap * torch.tanh(logits / cap)
    return (logits, layers) if return_layers else logits
