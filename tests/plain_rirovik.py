"""A plain, slow Rirovik in float64: whole sequences, no cache, one function per mechanism.

It shares no code with the package: configuration is read from the config.json dictionary as it
is, tensors by their checkpoint names.  Notation: x the residual stream [T, width], p the position
of a token in its sequence (from 0), H query heads, G shared key/value heads, c the key/value
latent of latent attention, r its turned key part.
"""

import math

import torch

F64 = torch.float64


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def squared_relu(z):
    z = torch.clamp(z, min=0.0)
    return z * z


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def layer_norm(x, stored, eps):
    """The layers' norm: its scale is stored as the distance from one."""
    return unit_rms(x, eps) * (1.0 + stored)


def turn(x, positions, rot):
    """x [T, heads, n]: of the first rot.dims channels (2i, 2i + 1) form pair i, rotated by p * base^(-2i / dims)."""
    dims, base = rot["dims"], rot["base"]
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=F64)
    angle = positions.to(F64)[:, None] * f[None, :]
    cos, sin = torch.cos(angle)[:, None, :], torch.sin(angle)[:, None, :]
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out = x.clone()
    out[..., 0:dims:2] = u * cos - v * sin
    out[..., 1:dims:2] = v * cos + u * sin
    return out


def visible(positions, mask):
    """[queries, keys]: earlier or equal, and near enough or among the kept first tokens."""
    distance = positions[:, None] - positions[None, :]
    seen = distance >= 0
    if mask and mask.get("size"):
        near = distance < mask["size"]
        kept = (positions < (mask.get("keep_first") or 0))[None, :]
        seen = seen & (near | kept)
    return seen


def softmax_over(scores, seen):
    scores = scores.masked_fill(~seen, -math.inf)
    e = torch.exp(scores - scores.max(-1, keepdim=True).values)
    return e / e.sum(-1, keepdim=True)


def attention(h, w, prefix, sizes, eps, latents=None):
    """Biased projections, unit query and key heads, no positions, a window that keeps the first tokens, a gate on
    every channel."""
    T = h.shape[0]
    H, G, D, V = sizes["heads"], sizes["kv_heads"], sizes["dim"], sizes["vdim"]
    project = lambda name: h @ w[prefix + name].T + w[prefix + name + ".b"]
    q = unit_rms(project("q").view(T, H, D), eps)
    k = unit_rms(project("k").view(T, G, D), eps)
    v = project("v").view(T, G, V)
    seen = visible(torch.arange(T), sizes.get("mask"))
    out = torch.zeros(T, H, V, dtype=F64)
    for head in range(H):
        shared = head // (H // G)
        out[:, head] = softmax_over((q[:, head] @ k[:, shared].T) * sizes["scale"], seen) @ v[:, shared]
    return (out.reshape(T, H * V) * sigmoid(h @ w[prefix + "g"].T)) @ w[prefix + "o"].T


def latent_of(h, w, prefix, sizes, eps):
    """(c [T, rank], r [T, rot_dim]): the normalised latent and the key part that all heads share, turned."""
    rank = sizes["kv_rank"]
    down = h @ w[prefix + "dkv"].T
    c = unit_rms(down[:, :rank], eps) * w[prefix + "dkv.norm"]
    r = down[:, None, rank:]
    if sizes["rot_dim"]:
        r = turn(r, torch.arange(h.shape[0]), dict(sizes["rot"], dims=sizes["rot_dim"]))
    return c, r[:, 0]


def latent_attention(h, w, prefix, sizes, eps, latents=None):
    """Queries through a normalised latent; keys and values from this layer's latent or an earlier layer's
    (`latents`: layer number -> (c, r), to which this layer adds its own under the key None)."""
    T = h.shape[0]
    H, D, R, V = sizes["heads"], sizes["dim"], sizes["rot_dim"], sizes["vdim"]
    positions = torch.arange(T)
    c_q = unit_rms(h @ w[prefix + "dq"].T, eps) * w[prefix + "dq.norm"]
    q = (c_q @ w[prefix + "uq"].T).view(T, H, D + R)
    q_plain, q_turned = q[..., :D], q[..., D:]
    if R:
        q_turned = turn(q_turned, positions, dict(sizes["rot"], dims=R))
    if sizes.get("kv_from") is not None:
        c, r = latents[sizes["kv_from"]]
    else:
        c, r = latents[None] = latent_of(h, w, prefix, sizes, eps)
    k_plain = (c @ w[prefix + "uk"].T).view(T, H, D)
    v = (c @ w[prefix + "uv"].T).view(T, H, V)
    seen = visible(positions, sizes.get("mask"))
    out = torch.zeros(T, H, V, dtype=F64)
    for head in range(H):
        scores = (q_plain[:, head] @ k_plain[:, head].T + q_turned[:, head] @ r.T) * sizes["scale"]
        out[:, head] = softmax_over(scores, seen) @ v[:, head]
    if prefix + "g" in w:
        out = out * sigmoid(h @ w[prefix + "g"].T)[:, :, None]
    return out.reshape(T, H * V) @ w[prefix + "o"].T


def unit(h, w, prefix):
    return squared_relu(h @ w[prefix + "up"].T) @ w[prefix + "down"].T


def choice(z, top):
    """(experts, weights): the largest logits, a softmax over those alone."""
    chosen = sorted(range(len(z)), key=lambda e: (-float(z[e]), e))[:top]
    e = torch.exp(z[chosen] - z[chosen].max())
    return chosen, e / e.sum()


def experts(h, w, prefix, mlp):
    z = h @ w[prefix + "router"].T + w[prefix + "router.b"]
    out = torch.zeros(h.shape[0], h.shape[1], dtype=F64)
    for t in range(h.shape[0]):
        for e, weight in zip(*choice(z[t], mlp["router"]["top"])):
            out[t] += weight * unit(h[t:t + 1], w, f"{prefix}e{e}.")[0]
    if mlp.get("shared"):
        out = out + unit(h, w, prefix + "shared.")
    return out


MIXERS = {"attention": attention, "latent_attention": latent_attention, "latent_attention_2": latent_attention}


def forward(ids, weights, config, streams=None):
    """float64 logits [T, vocab] of one whole sequence; `streams`, a list, receives the residual stream
    after every layer."""
    w = {name: tensor.to(F64) for name, tensor in weights.items()}
    eps = config["norm"]["eps"]
    x = w["embed"][torch.as_tensor(ids)] * config["embedding"]["scale"]
    latents = {}
    for index, layer in enumerate(config["layers"]):
        p = f"l{index}."
        y = MIXERS[layer["type"]](layer_norm(x, w[p + "norm1"], eps), w, p + "mix.", layer["mixer"], eps, latents)
        if None in latents:
            latents[index] = latents.pop(None)
        x = x + layer_norm(y, w[p + "norm1b"], eps)
        if layer.get("mlp") is not None:
            x = x + layer_norm(experts(layer_norm(x, w[p + "norm2"], eps), w, p + "mlp.", layer["mlp"]), w[p + "norm2b"], eps)
        if streams is not None:
            streams.append(x.clone())
    return layer_norm(x, w["final.norm"], eps) @ w["head"].T


def greedy(ids, weights, config, new_tokens):
    """The `new_tokens` tokens with the largest logit, each fed back."""
    ids, made = list(ids), []
    for _ in range(new_tokens):
        token = int(forward(ids, weights, config)[-1].argmax())
        made.append(token)
        ids.append(token)
    return made
