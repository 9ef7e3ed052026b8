"""A plain, slow Vipalorn in float64: one function a mechanism, whole sequences only, no cache and no kernels.

Written from the design's equations and shares nothing with the engine: the tests hold the engine's every way of
cutting a sequence against what these functions give for the sequence as a whole. ``w`` maps tensor names to float64
tensors, ``config`` is the dictionary a config.json holds.
"""

import torch


def layer_norm(x, w, eps):
    centred = x - x.mean(-1, keepdim=True)
    return centred / torch.sqrt((centred * centred).mean(-1, keepdim=True) + eps) * w


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def rotate(x, rot, first_position=0):
    """x ``[T, heads, width]``: the first rot.dims dimensions of a head turn by position, i paired with i + dims / 2."""
    dims = rot["dims"]
    half = dims // 2
    freq = rot["base"] ** (-2.0 * torch.arange(half, dtype=torch.float64) / dims)
    positions = torch.arange(first_position, first_position + x.shape[0], dtype=torch.float64)
    angle = (positions[:, None] * freq[None, :])[:, None, :]
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * torch.cos(angle) - v * torch.sin(angle), v * torch.cos(angle) + u * torch.sin(angle),
                      x[..., dims:]], dim=-1)


def causal_softmax(scores):
    """scores ``[heads, T, T]`` (query, key): softmax over the keys up to the query's own position."""
    T = scores.shape[-1]
    later = torch.arange(T)[None, :] > torch.arange(T)[:, None]
    return torch.softmax(scores.masked_fill(later, -float("inf")), dim=-1)


def latent_attention(w, p, m, h, eps):
    T = h.shape[0]
    H, d, r, rank = m["heads"], m["dim"], m["rot_dim"], m["kv_rank"]
    e = m.get("vdim", d)
    q = (h @ w[p + "q"].T).view(T, H, d + r)
    down = h @ w[p + "dkv"].T
    latent = rms_norm(down[:, :rank], w[p + "dkv.norm"], eps)
    shared = rotate(down[:, rank:].view(T, 1, r), m["rot"])[:, 0]
    turned = rotate(q[..., d:], m["rot"])
    keys = (latent @ w[p + "uk"].T).view(T, H, d)
    values = (latent @ w[p + "uv"].T).view(T, H, e)
    scores = torch.einsum("ihd,jhd->hij", q[..., :d], keys) + torch.einsum("ihd,jd->hij", turned, shared)
    out = torch.einsum("hij,jhd->ihd", causal_softmax(scores * m["scale"]), values)
    out = out * torch.sigmoid(h @ w[p + "g"].T)[:, :, None]                 # one gate a head
    return out.reshape(T, H * e) @ w[p + "o"].T


def short_convolution(u, w):
    """u ``[T, C]``, w ``[C, taps]``: y_t = sum_j w[:, j] u_(t - taps + 1 + j), zeros before the start."""
    taps = w.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=u.dtype), u])
    return sum(w[:, j] * padded[j:j + u.shape[0]] for j in range(taps))


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_rule_scan(q, k, v, beta, decay, state=None):
    """One head: q, k ``[T, d]``, v ``[T, e]``, beta and decay ``[T]``; returns outputs ``[T, e]`` and the state."""
    T, d = q.shape
    S = torch.zeros(d, v.shape[1], dtype=torch.float64) if state is None else state.clone()
    out = []
    for t in range(T):
        S = decay[t] * S
        u = beta[t] * (v[t] - S.T @ k[t])
        S = S + k[t][:, None] * u[None, :]
        out.append(S.T @ q[t])
    return torch.stack(out), S


def delta_mixer(w, p, m, h, eps):
    T = h.shape[0]
    H, d = m["heads"], m["dim"]
    G, e = m.get("kv_heads", H), m.get("vdim", d)
    silu = torch.nn.functional.silu
    q = silu(short_convolution(h @ w[p + "q"].T, w[p + "q.conv"])).view(T, G, d)
    k = silu(short_convolution(h @ w[p + "k"].T, w[p + "k.conv"])).view(T, G, d)
    v = silu(short_convolution(h @ w[p + "v"].T, w[p + "v.conv"])).view(T, H, e)
    q, k = unit(q) * d ** -0.5, unit(k)
    beta = torch.sigmoid(h @ w[p + "b"].T)
    step = torch.nn.functional.softplus(h @ w[p + "a"].T + w[p + "dt_bias"])
    decay = torch.exp(-torch.exp(w[p + "A_log"]) * step)                       # one a head
    gate = silu(h @ w[p + "g"].T).view(T, H, e)
    heads = []
    for head in range(H):
        source = head // (H // G)
        o, _ = delta_rule_scan(q[:, source], k[:, source], v[:, head], beta[:, head], decay[:, head])
        heads.append(rms_norm(o, w[p + "norm"], eps) * gate[:, head])
    return torch.cat(heads, dim=-1) @ w[p + "o"].T


def clipped_gate(gate, up, limit):
    g = torch.clamp(gate, max=limit)
    u = torch.clamp(up, -limit, limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1.0)


def expert(h, gate, up, down, limit):
    return clipped_gate(h @ gate.T, h @ up.T, limit) @ down.T


def route(z, top):
    """z ``[T, E]`` logits with their bias: the largest ``top`` (ties to the lower index) and the softmax over them."""
    order = torch.argsort(z, dim=-1, descending=True, stable=True)[:, :top]
    return order, torch.softmax(z.gather(1, order), dim=-1)


def routed_experts(w, p, m, h):
    limit, r = m["expert"]["limit"], m["router"]
    chosen, weights = route(h @ w[p + "router"].T + w[p + "router.b"], r["top"])
    out = torch.zeros_like(h)
    for e in range(r["experts"]):
        rows, slot = torch.nonzero(chosen == e, as_tuple=True)
        if rows.numel():
            y = expert(h[rows], *(w[f"{p}e{e}.{n}"] for n in ("gate", "up", "down")), limit)
            out.index_add_(0, rows, weights[rows, slot][:, None] * y)
    return out


def forward(config, w, tokens):
    """Logits ``[T, vocab]`` and the residual stream behind every layer ``[layers, T, width]``."""
    eps, mult = config["norm"]["eps"], config.get("residual_mult", 1.0)
    x = layer_norm(w["embed"][torch.tensor(tokens)], w["embed.norm"], eps)
    behind = []
    for i, layer in enumerate(config["layers"]):
        h = layer_norm(x, w[f"l{i}.norm1"], eps)                            # one norm, read by both sub-layers
        mixers = {"delta": delta_mixer, "latent_attention": latent_attention}
        y = mixers[layer["type"]](w, f"l{i}.mix.", layer["mixer"], h, eps)
        if layer.get("mlp"):
            y = y + routed_experts(w, f"l{i}.mlp.", layer["mlp"], h)
        x = x + mult * y
        behind.append(x)
    logits = layer_norm(x, w["final.norm"], eps) @ w["embed"].T * config.get("logit_scale", 1.0)
    return logits, torch.stack(behind)
