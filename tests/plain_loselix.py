"""A plain, slow Loselix in float64: whole sequences, no cache, one function per mechanism.

It shares no code with the package: configuration is read from the config.json dictionary as it
is, tensors by their checkpoint names.  Notation: x the residual stream [T, width], p the position
of a token in its sequence (from 0), H query heads on G key/value heads (query head h on key/value
head h // (H / G)), D a query's and key's head size, V a value's.
"""

import math

import torch

F64 = torch.float64


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def squared_relu(z):
    return torch.where(z > 0, z * z, torch.zeros_like(z))


def unit_rms(x, eps):
    """x over its root mean square (last axis, eps inside the root)."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def turn(x, positions, rot):
    """x [T, heads, n]: of every head the channels i and i + dims / 2 (i < dims / 2) are turned together by
    p * base^(-2i / dims); channels from dims on stay."""
    if not rot or not rot.get("dims"):
        return x
    dims, half = rot["dims"], rot["dims"] // 2
    f = torch.tensor([rot["base"] ** (-2.0 * i / dims) for i in range(half)], dtype=F64)
    angle = positions.to(F64)[:, None] * f[None, :]
    cos, sin = torch.cos(angle)[:, None, :], torch.sin(angle)[:, None, :]
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, x[..., dims:]], dim=-1)


def softcap(scores, cap):
    """A smooth bound on the scores: cap tanh(s / cap)."""
    return cap * torch.tanh(scores / cap) if cap else scores


def softmax_over(scores, seen):
    scores = scores.masked_fill(~seen, -math.inf)
    e = torch.exp(scores - scores.max(-1, keepdim=True).values)
    return e / e.sum(-1, keepdim=True)


def sigmoid_over(scores, seen, bias):
    """Every visible key's own weight sigmoid(s + bias); nothing is normalised over the keys."""
    return torch.where(seen, sigmoid(scores + bias), torch.zeros_like(scores))


def causal(T):
    p = torch.arange(T)
    return p[:, None] >= p[None, :]


def temperature(positions, coef, every):
    """1 + coef ln(floor((p + 1) / every) + 1): queries grow sharper with their position."""
    steps = (positions + 1) // every
    return 1.0 + coef * torch.log(steps.to(F64) + 1.0)


def difference_weight(w, prefix, diff):
    """lambda = exp(lq1 . lk1) - exp(lq2 . lk2) + diff."""
    first = math.exp(float((w[prefix + "lq1"] * w[prefix + "lk1"]).sum()))
    second = math.exp(float((w[prefix + "lq2"] * w[prefix + "lk2"]).sum()))
    return first - second + diff


def differential_attention(h, w, prefix, sizes, eps):
    """Two softmax maps a head over the same values, the second taken off the first with weight lambda; the
    difference over its root mean square, times 1 - diff."""
    T = h.shape[0]
    H, G, D, V = sizes["heads"], sizes["kv_heads"], sizes["dim"], sizes["vdim"]
    positions, seen = torch.arange(T), causal(T)
    q = turn((h @ w[prefix + "q"].T).view(T, 2 * H, D), positions, sizes.get("rot")).view(T, H, 2, D)
    k = turn((h @ w[prefix + "k"].T).view(T, 2 * G, D), positions, sizes.get("rot")).view(T, G, 2, D)
    v = (h @ w[prefix + "v"].T).view(T, G, V)
    lam = difference_weight(w, prefix, sizes["diff"])
    out = torch.zeros(T, H, V, dtype=F64)
    for head in range(H):
        shared = head // (H // G)
        maps = [softmax_over(softcap((q[:, head, m] @ k[:, shared, m].T) * sizes["scale"], sizes.get("softcap")), seen)
                @ v[:, shared] for m in (0, 1)]
        out[:, head] = unit_rms(maps[0] - lam * maps[1], eps) * (1.0 - sizes["diff"])
    return out.reshape(T, H * V) @ w[prefix + "o"].T


def head_gated_attention(h, w, prefix, sizes, eps):
    """Softmax attention whose heads' outputs are each multiplied by one number, sigmoid(W_g h)."""
    T = h.shape[0]
    H, G, D, V = sizes["heads"], sizes["kv_heads"], sizes["dim"], sizes["vdim"]
    positions, seen = torch.arange(T), causal(T)
    q = turn((h @ w[prefix + "q"].T).view(T, H, D), positions, sizes.get("rot"))
    k = turn((h @ w[prefix + "k"].T).view(T, G, D), positions, sizes.get("rot"))
    v = (h @ w[prefix + "v"].T).view(T, G, V)
    gate = sigmoid(h @ w[prefix + "g"].T)                                     # [T, H]
    out = torch.zeros(T, H, V, dtype=F64)
    for head in range(H):
        shared = head // (H // G)
        out[:, head] = softmax_over((q[:, head] @ k[:, shared].T) * sizes["scale"], seen) @ v[:, shared] * gate[:, head:head + 1]
    return out.reshape(T, H * V) @ w[prefix + "o"].T


def sigmoid_attention(h, w, prefix, sizes, eps):
    """Keys' weights without a softmax; the values are the projected keys before their norm; no rotation, but
    queries that grow with their position; a gate on every channel."""
    T = h.shape[0]
    H, G, D = sizes["heads"], sizes["kv_heads"], sizes["dim"]
    positions, seen = torch.arange(T), causal(T)
    k_rows = h @ w[prefix + "k"].T
    q = (unit_rms(h @ w[prefix + "q"].T, eps) * w[prefix + "q.norm"]).view(T, H, D)
    k = (unit_rms(k_rows, eps) * w[prefix + "k.norm"]).view(T, G, D)
    v = k_rows.view(T, G, D)
    if sizes.get("q_temp"):
        q = q * temperature(positions, sizes["q_temp"]["coef"], sizes["q_temp"]["every"])[:, None, None]
    out = torch.zeros(T, H, D, dtype=F64)
    for head in range(H):
        shared = head // (H // G)
        out[:, head] = sigmoid_over((q[:, head] @ k[:, shared].T) * sizes["scale"], seen, w[prefix + "pb"][head]) @ v[:, shared]
    out = out.reshape(T, H * D) * sigmoid(h @ w[prefix + "g"].T)
    return out @ w[prefix + "o"].T


def feed_forward(h, w, prefix):
    return squared_relu(h @ w[prefix + "up"].T) @ w[prefix + "down"].T


MIXERS = {"attention": differential_attention, "attention_2": head_gated_attention, "attention_3": sigmoid_attention}


def runs(config):
    """[(layer, whether the embedding's output joins the stream before it)] in the order the layers run."""
    count, loop = len(config["layers"]), config.get("loop")
    if not loop:
        return [(i, False) for i in range(count)]
    order = [(i, False) for i in range(loop["start"])]
    for turn_number in range(loop["times"]):
        order += [(i, turn_number > 0 and i == loop["start"]) for i in range(loop["start"], loop["stop"])]
    return order + [(i, False) for i in range(loop["stop"], count)]


def forward(ids, weights, config, streams=None):
    """float64 logits [T, vocab] of one whole sequence; `streams`, a list, receives the residual stream
    after every run of a layer."""
    w = {name: tensor.to(F64) for name, tensor in weights.items()}
    eps = config["norm"]["eps"]
    origin = w["embed"][torch.as_tensor(ids)]
    x = origin.clone()
    for index, enters_again in runs(config):
        if enters_again:
            x = x + origin
        layer, p = config["layers"][index], f"l{index}."
        h = unit_rms(x, eps) * w[p + "norm1"]
        out = MIXERS[layer["type"]](h, w, p + "mix.", layer["mixer"], eps)
        if layer.get("mlp") is not None:
            out = out + feed_forward(h, w, p + "mlp.")
        x = x + out
        if streams is not None:
            streams.append(x.clone())
    return unit_rms(x, eps) * w["final.norm"] @ w["head"].T


def greedy(ids, weights, config, new_tokens):
    """The `new_tokens` tokens with the largest logit, each fed back."""
    ids, made = list(ids), []
    for _ in range(new_tokens):
        token = int(forward(ids, weights, config)[-1].argmax())
        made.append(token)
        ids.append(token)
    return made
