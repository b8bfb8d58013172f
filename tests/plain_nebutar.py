"""A plain, slow Nebutar in PyTorch: one whole sequence from position 0, no cache, no batches.

It is the oracle the framework's Nebutar is compared with, written from the design's equations with
one function per mechanism, and shares no code with ``socrates_amd``. ``w`` maps tensor names to
tensors (any float dtype; everything is computed in the dtype of ``x``, float64 in the tests),
``cfg`` is the dict of ``config.json``.

Notation: T tokens, d the model's width, H heads, G key heads. A linear weight W is stored [out, in]
and applied as x @ W.T.
"""

import torch


# ---- norms ------------------------------------------------------------------------------------
def layer_norm(x, weight, bias, eps):
    c = x - x.mean(-1, keepdim=True)
    return c / torch.sqrt(c.pow(2).mean(-1, keepdim=True) + eps) * weight + bias


def over_rms(x, eps):
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def unit(x, eps=1e-6):
    return x / torch.sqrt(x.pow(2).sum(-1, keepdim=True) + eps)


def silu(x):
    return x * torch.sigmoid(x)


# ---- attention inside fixed chunks of positions -------------------------------------------------
def chunk_mask(T, chunk):
    """[T, T] bool: query i (row) sees key j."""
    i, j = torch.arange(T).view(-1, 1), torch.arange(T).view(1, -1)
    return (j <= i) & (i // chunk == j // chunk)


def chunked_attention(h, w, p, m):
    T, H, G, D, Dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T).view(T, H, D)
    k = (h @ w[p + "k"].T).view(T, G, D).repeat_interleave(H // G, dim=1)
    v = (h @ w[p + "v"].T).view(T, G, Dv).repeat_interleave(H // G, dim=1)
    s = torch.einsum("ihd,jhd->hij", q, k) * m["scale"]
    s = m["softcap"] * torch.tanh(s / m["softcap"])
    s = s.masked_fill(~chunk_mask(T, m["mask"]["size"]), float("-inf"))
    o = torch.einsum("hij,jhd->ihd", torch.softmax(s, dim=-1), v)
    return o.reshape(T, H * Dv) @ w[p + "o"].T


# ---- gated delta rule -----------------------------------------------------------------------------
def causal_conv(x, taps):
    """x [T, C], taps [C, n]: the last tap is the current token's, zeros before the start."""
    T, n = x.shape[0], taps.shape[1]
    padded = torch.cat([torch.zeros(n - 1, x.shape[1], dtype=x.dtype), x])
    return sum(padded[j:j + T] * taps[:, j] for j in range(n))


def delta_walk(q, k, v, g, beta, state=None):
    """q, k [T, H, D], v [T, H, Dv], g, beta [T, H]: per head and token S <- g S; u = beta (v - S^T k);
    S <- S + k u^T; o = S^T q. Returns (o [T, H, Dv], the last S [H, D, Dv])."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype) if state is None else state.clone()
    out = torch.empty_like(v)
    for t in range(T):
        S = g[t].view(H, 1, 1) * S
        u = beta[t].view(H, 1) * (v[t] - (S * k[t].unsqueeze(-1)).sum(1))          # S^T k, head by head
        S = S + k[t].unsqueeze(-1) * u.unsqueeze(1)
        out[t] = (S * q[t].unsqueeze(-1)).sum(1)
    return out, S


def delta_inputs(h, w, p, m):
    """(q, k, v, g, beta) as the walk takes them."""
    T, H, G, D, Dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(causal_conv(h @ w[p + n].T, w[p + n + ".conv"])) for n in "qkv")
    q = (unit(q.view(T, G, D)) * D ** -0.5).repeat_interleave(H // G, dim=1)
    k = unit(k.view(T, G, D)).repeat_interleave(H // G, dim=1)
    beta = torch.sigmoid(h @ w[p + "b"].T)
    step = torch.nn.functional.softplus(h @ w[p + "a"].T + w[p + "dt_bias"], threshold=1e9)
    g = torch.exp(-torch.exp(w[p + "A_log"]) * step)
    return q, k, v.view(T, H, Dv), g, beta


def delta_mixer(h, w, p, m, eps):
    o, _ = delta_walk(*delta_inputs(h, w, p, m))
    o = over_rms(o, eps) * w[p + "norm"]
    return (o.reshape(h.shape[0], -1) * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


# ---- both side by side ------------------------------------------------------------------------------
def parallel_mixer(h, w, p, m, eps):
    return (m["left_scale"] * chunked_attention(h, w, p + "left.", m["left"])
            + m["right_scale"] * delta_mixer(h, w, p + "right.", m["right"], eps))


# ---- experts, some of which hand their input through ---------------------------------------------------
def expert(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def router(h, w, p, top):
    """(experts [T, top], weights [T, top]): chosen by softmax score + correction, weighted by the score."""
    s = torch.softmax(h @ w[p + "router"].T, dim=-1)
    chosen = (s + w[p + "correction"]).topk(top, dim=-1).indices
    return chosen, s.gather(-1, chosen)


def experts_mixture(h, w, p, mlp):
    experts, weights = router(h, w, p, mlp["router"]["top"])
    E = mlp["router"]["experts"]
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, a in zip(experts[t].tolist(), weights[t]):
            out[t] = out[t] + a * (h[t] if e >= E else expert(h[t:t + 1], w, f"{p}e{e}.")[0])
    return out


# ---- several copies of the stream ---------------------------------------------------------------------------
def through_streams(x, w, p, sublayer):
    """x [s, T, d]: u = sum_a in[a] x_a, y = sublayer(u), x_b <- sum_a mix[a, b] x_a + out[b] y."""
    y = sublayer(torch.einsum("a,atd->td", w[p + "in"], x))
    return torch.einsum("ab,atd->btd", w[p + "mix"], x) + w[p + "out"].view(-1, 1, 1) * y


# ---- the model ----------------------------------------------------------------------------------------
def run_order(cfg):
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return list(range(n))
    body = list(range(loop["start"], loop["stop"]))
    return list(range(loop["start"])) + body * loop["times"] + list(range(loop["stop"], n))


def forward(cfg, w, ids, trace=None):
    """Logits [T, vocab] of the whole sequence ``ids``. ``trace``: a list that receives the sum of the
    streams after every layer run."""
    eps = cfg["norm"]["eps"]
    e = w["embed"][torch.as_tensor(ids, dtype=torch.long)] * cfg["embedding"]["scale"] + w["pos"][:len(ids)]
    x = e.unsqueeze(0).repeat(cfg["streams"], 1, 1)
    for i in run_order(cfg):
        L, layer = f"l{i}.", cfg["layers"][i]
        x = through_streams(x, w, L + "hc1.", lambda u: parallel_mixer(
            layer_norm(u, w[L + "norm1"], w[L + "norm1.b"], eps), w, L + "mix.", layer["mixer"], eps))
        if layer.get("mlp") is not None:
            x = through_streams(x, w, L + "hc2.", lambda u: experts_mixture(
                layer_norm(u, w[L + "norm2"], w[L + "norm2.b"], eps), w, L + "mlp.", layer["mlp"]))
        if trace is not None:
            trace.append(x.sum(0))
    return layer_norm(x.sum(0), w["final.norm"], w["final.norm.b"], eps) @ w["embed"].T


def greedy(cfg, w, prompt, n_new):
    ids = list(prompt)
    for _ in range(n_new):
        ids.append(int(forward(cfg, w, ids)[-1].argmax()))
    return ids[len(prompt):]
