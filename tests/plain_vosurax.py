"""A plain, slow Vosurax in float64: one function a mechanism, whole sequences only, no cache and no kernels.

Written from the design's equations and shares nothing with the engine: the tests hold the engine's every way of
cutting a sequence against what these functions give for the sequence as a whole. ``w`` maps tensor names to float64
tensors, ``config`` is the dictionary a config.json holds.
"""

import math

import torch


def over_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def stream_norm(x, w, eps):
    """The weight is stored around zero."""
    return over_rms(x, eps) * (1.0 + w)


def rotate(x, rot, first_position=0):
    """x ``[T, heads, width]``: the first rot.dims dimensions of a head turn by position, i paired with i + dims / 2."""
    dims = rot.get("dims", x.shape[-1])
    half = dims // 2
    freq = rot["base"] ** (-2.0 * torch.arange(half, dtype=torch.float64) / dims)
    positions = torch.arange(first_position, first_position + x.shape[0], dtype=torch.float64)
    angle = (positions[:, None] * freq[None, :])[:, None, :]
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * torch.cos(angle) - v * torch.sin(angle), v * torch.cos(angle) + u * torch.sin(angle),
                      x[..., dims:]], dim=-1)


def seen_in_chunks(T, size):
    """bool ``[T, T]`` (query, key): earlier or own position, same chunk of ``size`` positions counted from 0."""
    i = torch.arange(T)
    same = torch.ones(T, T, dtype=torch.bool) if size is None else i[:, None] // size == i[None, :] // size
    return same & (i[None, :] <= i[:, None])


def chunked_attention(w, p, m, h, eps):
    T = h.shape[0]
    H, d = m["heads"], m["dim"]
    G, e = m.get("kv_heads", H), m.get("vdim", d)
    q = (h @ w[p + "q"].T + w[p + "q.b"]).view(T, H, d)
    k = (h @ w[p + "k"].T + w[p + "k.b"]).view(T, G, d)
    v = (h @ w[p + "v"].T + w[p + "v.b"]).view(T, G, e)
    q = over_rms(q, eps) * w[p + "q.norm"]
    k = over_rms(k, eps) * w[p + "k.norm"]
    seen = seen_in_chunks(T, (m.get("mask") or {}).get("size"))
    heads = []
    for head in range(H):
        source = head // (H // G)
        scores = (q[:, head] @ k[:, source].T * m["scale"]).masked_fill(~seen, -float("inf"))
        heads.append(torch.softmax(scores, dim=-1) @ v[:, source])
    gate = torch.sigmoid(h @ w[p + "g"].T)
    return (torch.cat(heads, dim=-1) * gate) @ w[p + "o"].T


def matrix_memory_scan(q, k, v, log_in, log_forget, state=None):
    """One head: q (already scaled), k ``[T, d]``, v ``[T, e]``, the logarithms of the gates ``[T]``; returns outputs
    ``[T, e]`` and the state (S, n, m)."""
    T, d = q.shape
    if state is None:
        S, n, m = torch.zeros(d, v.shape[1], dtype=torch.float64), torch.zeros(d, dtype=torch.float64), 0.0
    else:
        S, n, m = state
    out = []
    for t in range(T):
        f, i = float(log_forget[t]), float(log_in[t])
        old, m = m, max(f + m, i)
        keep, take = math.exp(f + old - m), math.exp(i - m)
        S = keep * S + take * k[t][:, None] * v[t][None, :]
        n = keep * n + take * k[t]
        out.append(S.T @ q[t] / (max(abs(float(n @ q[t])), math.exp(-m)) + 1e-6))
    return torch.stack(out), (S, n, m)


def capped(z, cap):
    return cap * torch.tanh(z / cap)


def matrix_memory(w, p, m, h, eps):
    T = h.shape[0]
    H, d, e, cap = m["heads"], m["dim"], m.get("vdim", m["dim"]), m["gate_cap"]
    q = (h @ w[p + "q"].T).view(T, H, d) * d ** -0.5
    k = (h @ w[p + "k"].T).view(T, H, d)
    v = (h @ w[p + "v"].T).view(T, H, e)
    log_in = capped(h @ w[p + "i"].T + w[p + "i.b"], cap)
    log_forget = torch.nn.functional.logsigmoid(capped(h @ w[p + "f"].T + w[p + "f.b"], cap))
    heads = [over_rms(matrix_memory_scan(q[:, j], k[:, j], v[:, j], log_in[:, j], log_forget[:, j])[0], eps)
             for j in range(H)]
    return (torch.cat(heads, dim=-1) * w[p + "norm"] * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def parallel_mixer(w, p, m, h, eps):
    left = chunked_attention(w, p + "left.", m["left"], h, eps)
    right = matrix_memory(w, p + "right.", m["right"], h, eps)
    return 0.5 * (over_rms(left, eps) * w[p + "left.out"] + over_rms(right, eps) * w[p + "right.out"])


def retention_scan(q, k, v, decay, state=None):
    """One head: q, k ``[T, d]`` (k already scaled), v ``[T, e]``, one decay; returns outputs ``[T, e]`` and the state."""
    S = torch.zeros(q.shape[1], v.shape[1], dtype=torch.float64) if state is None else state
    out = []
    for t in range(q.shape[0]):
        S = decay * S + k[t][:, None] * v[t][None, :]
        out.append(S.T @ q[t])
    return torch.stack(out), S


def retention_mixer(w, p, m, h, eps):
    T = h.shape[0]
    H, d = m["heads"], m["dim"]
    e = m.get("vdim", d)
    q = rotate((h @ w[p + "q"].T).view(T, H, d), m["rot"])
    k = rotate((h @ w[p + "k"].T).view(T, H, d), m["rot"]) * d ** -0.5
    v = (h @ w[p + "v"].T).view(T, H, e)
    heads = [over_rms(retention_scan(q[:, j], k[:, j], v[:, j], m["decay"][j])[0], eps) for j in range(H)]
    return (torch.cat(heads, dim=-1) * torch.nn.functional.silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def dense(w, p, h):
    return gelu_tanh(h @ w[p + "up"].T) @ w[p + "down"].T


def expert(h, gate, up, down):
    return (torch.nn.functional.silu(h @ gate.T) * (h @ up.T)) @ down.T


def route(z, top):
    """z ``[T, E]`` logits: the ``top`` largest (ties to the lower index) and their sigmoids, as they are."""
    scores = torch.sigmoid(z)
    order = torch.argsort(scores, dim=-1, descending=True, stable=True)[:, :top]
    return order, scores.gather(1, order)


def routed_experts(w, p, m, h):
    chosen, weights = route(h @ w[p + "router"].T, m["router"]["top"])
    out = torch.zeros_like(h)
    for e in range(m["router"]["experts"]):
        rows, slot = torch.nonzero(chosen == e, as_tuple=True)
        if rows.numel():
            x = weights[rows, slot][:, None] * h[rows]                   # the weight is on the input
            out.index_add_(0, rows, expert(x, *(w[f"{p}e{e}.{n}"] for n in ("gate", "up", "down"))))
    if m.get("shared"):
        out = out + expert(h, *(w[f"{p}shared.{n}"] for n in ("gate", "up", "down")))
    return out


def run_order(config):
    """(layer, number of the pass if the layer opens one, else None), in the order the layers run."""
    n = len(config["layers"])
    loop = config.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    start, stop = loop["start"], loop["stop"]
    order = [(i, None) for i in range(start)]
    for t in range(loop["times"]):
        order += [(i, t if i == start else None) for i in range(start, stop)]
    return order + [(i, None) for i in range(stop, n)]


def layer_forward(config, w, i, x):
    eps, layer, p = config["norm"]["eps"], config["layers"][i], f"l{i}."
    mixer = {"parallel": parallel_mixer, "retention": retention_mixer}[layer["type"]]
    x = x + mixer(w, p + "mix.", layer["mixer"], stream_norm(x, w[p + "norm1"], eps), eps)
    mlp = layer.get("mlp")
    if mlp:
        h = stream_norm(x, w[p + "norm2"], eps)
        x = x + (dense(w, p + "mlp.", h) if mlp["kind"] == "dense" else routed_experts(w, p + "mlp.", mlp, h))
    return x


def forward(config, w, tokens):
    """Logits ``[T, vocab]`` and the residual stream behind every layer run ``[runs, T, width]``."""
    x = w["embed"][torch.tensor(tokens)]
    behind = []
    for i, opens in run_order(config):
        if opens is not None:
            x = x + w["loop.step"][opens]
        x = layer_forward(config, w, i, x)
        behind.append(x)
    return stream_norm(x, w["final.norm"], config["norm"]["eps"]) @ w["head"].T, torch.stack(behind)
