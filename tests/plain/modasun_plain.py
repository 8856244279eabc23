"""Modasun, plainly: whole sequences, no cache, no batch, one function a mechanism.

A decoder whose layers norm the sum of a weighed stream and a sublayer's result,

    x = norm1(alpha x + mixer(x));   x = norm2(alpha x + ff(x))        (ff may be absent)
    norm(v) = v / sqrt(mean(v^2) + eps) * (1 + w)

The mixer is, layer by layer,

  "attention": causal softmax attention with grouped key/value heads and no rotation; every query and key head is
      divided by its root mean square, and a query is multiplied by a temperature that grows with the logarithm of
      its position;
  "channel_delta": a gated delta rule, S = diag(g) S, S += k (beta (v - S^T k))^T, o = S^T q, whose decay g is a
      number a head and key channel, with short convolutions on q, k and v, unit queries and keys, and a gated norm.

The feed-forward is W_down relu(W_up x)^2, or a mixture of silu-gated experts chosen by sigmoid scores plus a
correction among the experts of the best groups (a group's score: the sum of its two best), with a shared expert
that enters by a gate of its own.  A layer may use another layer's weights.  The head is the embedding table.

Every function takes and returns tensors of one dtype (float64 in the tests' reference runs); `rounding` is a
function applied wherever a bfloat16 model would hold a tensor in bfloat16, and the identity otherwise.  Nothing
here is shared with the engine.
"""
from __future__ import annotations

import torch


def same(x):
    return x


def silu(z):
    return z * torch.sigmoid(z)


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def offset_norm(x, weight, eps):
    return unit_rms(x, eps) * (1.0 + weight)


def norm_of_the_sum(x, y, alpha, weight, eps):
    return offset_norm(alpha * x + y, weight, eps)


def query_temperature(positions, coef, every):
    """1 + coef ln(floor((p + 1) / every) + 1)."""
    return 1.0 + coef * torch.log(torch.div(positions + 1, every, rounding_mode="floor") + 1.0)


def causal_softmax(scores):
    T = scores.shape[-1]
    seen = torch.arange(T)[:, None] >= torch.arange(T)[None, :]
    scores = scores.masked_fill(~seen, float("-inf"))
    e = torch.exp(scores - scores.max(dim=-1, keepdim=True).values)
    return e / e.sum(dim=-1, keepdim=True)


def attention(h, w, p, c, eps, rounding=same):
    T = h.shape[0]
    H, G, d, dv = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    q = unit_rms(rounding(h @ w[p + "q"].T).view(T, H, d), eps)
    k = rounding(unit_rms(rounding(h @ w[p + "k"].T).view(T, G, d), eps))
    v = rounding(h @ w[p + "v"].T).view(T, G, dv)
    if c.get("q_temp") is not None:
        temp = query_temperature(torch.arange(T).to(h.dtype), c["q_temp"]["coef"], c["q_temp"]["every"])
        q = q * temp[:, None, None]
    q = rounding(q)
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for head in range(H):
        g = head // (H // G)
        out[:, head] = causal_softmax(q[:, head] @ k[:, g].T * c["scale"]) @ v[:, g]
    return rounding(rounding(out.reshape(T, H * dv)) @ w[p + "o"].T)


def short_convolution(z, taps_weight):
    """z [T, C], taps_weight [C, taps]: sum_j w[:, j] z_(t - taps + 1 + j), zeros before the start, then silu."""
    T, C = z.shape
    taps = taps_weight.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, C, dtype=z.dtype), z], dim=0)
    out = torch.zeros_like(z)
    for j in range(taps):
        out = out + taps_weight[:, j] * padded[j:j + T]
    return silu(out)


def unit_vector(x):
    return x / torch.sqrt((x * x).sum(dim=-1, keepdim=True) + 1e-6)


def channel_decay(z, a_log, dt_bias):
    """z [T, H, d] -> exp(-exp(a_log) softplus(z + dt_bias)), a number a head and channel."""
    dt = torch.nn.functional.softplus(z + dt_bias, threshold=1e9)
    return torch.exp(-torch.exp(a_log)[:, None] * dt)


def delta_rule(q, k, v, g, beta):
    """Token by token; q, k, g [T, H, d], v [T, H, dv], beta [T, H] -> o [T, H, dv]."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=q.dtype)
    out = torch.zeros_like(v)
    for t in range(T):
        S = g[t][:, :, None] * S
        seen = (S * k[t][:, :, None]).sum(1)
        u = beta[t][:, None] * (v[t] - seen)
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


def channel_delta(h, w, p, c, eps, rounding=same):
    T = h.shape[0]
    H, G, d, dv = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    q, k, v = (rounding(short_convolution(rounding(h @ w[p + n].T), w[f"{p}{n}.conv"])) for n in "qkv")
    q = unit_vector(q.view(T, G, d)).repeat_interleave(H // G, dim=1) * d ** -0.5
    k = unit_vector(k.view(T, G, d)).repeat_interleave(H // G, dim=1)
    beta = torch.sigmoid(rounding(h @ w[p + "b"].T))
    z = rounding(rounding(h @ w[p + "a1"].T) @ w[p + "a2"].T)
    g = channel_decay(z.view(T, H, d), w[p + "A_log"], w[p + "dt_bias"].view(H, d))
    o = delta_rule(q, k, v.view(T, H, dv), g, beta)
    gate = torch.sigmoid(rounding(rounding(h @ w[p + "g1"].T) @ w[p + "g2"].T)).view(T, H, dv)
    o = unit_rms(o, eps) * w[p + "norm"] * gate
    return rounding(rounding(o.reshape(T, H * dv)) @ w[p + "o"].T)


def squared_relu(z):
    return torch.clamp(z, min=0.0) ** 2


def dense_feed_forward(h, w, p, rounding=same):
    return rounding(rounding(squared_relu(rounding(h @ w[p + "up"].T))) @ w[p + "down"].T)


def gated_feed_forward(h, w, p, rounding=same):
    return rounding(silu(rounding(h @ w[p + "gate"].T)) * rounding(h @ w[p + "up"].T)) @ w[p + "down"].T


def choose_experts(z, correction, top, groups=1, keep=1):
    """z [E], the router's logits -> (the chosen experts, their weights)."""
    s = torch.sigmoid(z)
    choice = s + correction
    per = len(z) // groups
    by_group = [sum(sorted(choice[g * per:(g + 1) * per].tolist())[-2:]) for g in range(groups)]
    kept = sorted(range(groups), key=lambda g: -by_group[g])[:keep]
    allowed = [e for e in range(len(z)) if e // per in kept]
    chosen = sorted(allowed, key=lambda e: -choice[e].item())[:top]
    return chosen, s[chosen] / (s[chosen].sum() + 1e-20)


def expert_feed_forward(h, w, p, c, rounding=same):
    r = c["router"]
    groups = r.get("groups") or {"count": 1, "keep": 1}
    z = h @ w[p + "router"].T
    out = torch.zeros(h.shape[0], w[p + "e0.down"].shape[0], dtype=h.dtype)
    used = {}
    for t in range(h.shape[0]):
        for e, weight in zip(*choose_experts(z[t], w[p + "correction"], r["top"], groups["count"], groups["keep"])):
            used.setdefault(e, []).append((t, weight))
    for e, tokens in used.items():
        at = [t for t, _ in tokens]
        out[at] += torch.stack([x for _, x in tokens])[:, None] * gated_feed_forward(h[at], w, f"{p}e{e}.", rounding)
    if c.get("shared") is not None:
        opened = torch.sigmoid(rounding(h @ w[p + "shared.sg"].T))
        out = out + opened * gated_feed_forward(h, w, p + "shared.", rounding)
    return out


MIXERS = {"attention": attention, "channel_delta": channel_delta}


def weights_layer(cfg, i):
    """The layer whose tensors layer i uses."""
    while cfg["layers"][i].get("weights_of") is not None:
        i = cfg["layers"][i]["weights_of"]
    return i


def forward(tokens, w, cfg, rounding=same, keep_layers=False):
    """tokens: a list of ids; w: {name: tensor}; cfg: config.json as a dict.  Returns logits [T, vocab] (and the
    stream after every layer)."""
    eps, alpha = cfg["norm"]["eps"], cfg["postln_alpha"]
    x = w["embed"][torch.as_tensor(tokens)] * cfg["embedding"]["scale"]
    after = []
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{weights_layer(cfg, i)}."
        y = MIXERS[layer["type"]](rounding(x), w, p + "mix.", layer["mixer"], eps, rounding)
        x = norm_of_the_sum(x, y, alpha, w[p + "norm1"], eps)
        mlp = layer.get("mlp")
        if mlp is not None:
            if mlp["kind"] == "dense":
                y = dense_feed_forward(rounding(x), w, p + "mlp.", rounding)
            else:
                y = expert_feed_forward(rounding(x), w, p + "mlp.", mlp, rounding)
            x = norm_of_the_sum(x, y, alpha, w[p + "norm2"], eps)
        after.append(x)
    logits = rounding(offset_norm(x, w["final.norm"], eps)) @ w["embed"].T
    return (logits, torch.stack(after)) if keep_layers else logits
