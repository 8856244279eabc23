"""Shared by the Modasun tests: small configurations that differ in every size and option, model folders whose weights
make every mechanism count, and the comparison with the plain implementation."""
from __future__ import annotations

import copy
import hashlib
import json
import os
import random

import torch

from duvozen_helpers import read_folder, to_bfloat16  # noqa: F401  (a folder is read the same way)
from lefisun_helpers import compare_with_rounding  # noqa: F401  (the comparison is the same)
from plain import modasun_plain
from tokuvik_helpers import compare_rows, random_ids  # noqa: F401
from wllm_amd.parts import build_model
from wllm_amd.weights.safetensors_io import write_safetensors


def attention(heads, kv_heads, dim, vdim, *, scale=None, temp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale if scale is not None else dim ** -0.5}
    if temp is not None:
        m["q_temp"] = {"coef": temp[0], "every": temp[1]}
    return "attention", m


def delta(heads, kv_heads, dim, vdim, taps):
    return "channel_delta", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": taps}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def experts(ff, count, top, *, groups=None, shared=None):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": count, "top": top}}
    if groups is not None:
        m["router"]["groups"] = {"count": groups[0], "keep": groups[1]}
    if shared is not None:
        m["shared"] = {"ff": shared}
    return m


def layer(mixer, mlp, weights_of=None):
    entry = {"type": mixer[0], "mixer": mixer[1], "mlp": mlp}
    if weights_of is not None:
        entry["weights_of"] = weights_of
    return entry


def config(vocab, width, layers, *, scale=1.0, alpha=1.0, eps=1e-6):
    return {"architecture": "Modasun", "vocab": vocab, "width": width, "embedding": {"scale": scale}, "norm": {"eps": eps},
            "postln_alpha": alpha, "layers": layers}


def again(layers, j):
    """One more run of layer j's weights."""
    return {**copy.deepcopy(layers[j]), "weights_of": j}


# A recurrence first, more value heads than key heads, heads the matrix cores take, values narrower and wider than keys,
# a temperature that passes many steps within a request, one without any, layers without a feed-forward, both mixers run
# again (a run of a run among them), groups of which two or all are kept, a top of one and of three.
_MIXED = [
    layer(delta(4, 2, 16, 32, 4), experts(32, 8, 3, groups=(4, 2), shared=48)),
    layer(attention(4, 2, 32, 16, scale=0.4, temp=(0.5, 9)), dense(96)),
    layer(attention(2, 1, 64, 32), None),
    layer(delta(2, 2, 32, 16, 3), dense(64)),
]
MIXED = dict(page_size=16, seed=51, inner={0: (12, 20), 3: (8, 5)}, config=config(160, 64, _MIXED + [
    again(_MIXED, 0), again(_MIXED, 1), layer(attention(4, 4, 32, 32, temp=(-0.2, 40)), experts(48, 6, 1, groups=(2, 2))),
    {**again(_MIXED, 0), "weights_of": 4}], scale=2.0, alpha=1.5, eps=1e-5))

# Sizes no matrix-core kernel takes and no vector of four fits (heads of 20, 10 and 7 channels, a width of 48, feed-forwards
# of odd sizes, pages of 8), as many key heads as query heads, one head, one expert, groups of one expert each, a top of
# all experts, one tap and many, a head of more channels than a wavefront, inner sizes of one and of many.
ODD = dict(page_size=8, seed=52, inner={1: (1, 30), 2: (40, 3), 4: (7, 7)}, config=config(97, 48, [
    layer(attention(3, 3, 20, 28, scale=0.9, temp=(1.0, 1)), experts(24, 5, 5, shared=9)),
    layer(delta(3, 1, 10, 6, 1), dense(37)),
    layer(delta(1, 1, 130, 5, 7), experts(56, 1, 1)),
    layer(attention(5, 1, 12, 8, scale=0.5, temp=(0.7, 1000)), experts(30, 4, 2, groups=(4, 3), shared=30)),
    layer(delta(4, 2, 7, 9, 2), None),
    layer(attention(1, 1, 6, 3, scale=0.6), dense(40)),
], scale=0.7, alpha=0.6, eps=1e-6))

# Attention so sharp that single keys decide, decays from nearly nothing to nearly one within one head, step sizes from
# nothing to one, corrections that outweigh the scores, a strong stream: a key lost or gained, a stale slot, a wrong page, a
# lost state or carried row moves the logits by far more than rounding.
SHARP = dict(page_size=16, seed=53, sharp=True, inner={1: (16, 16), 3: (24, 8)}, config=config(200, 96, [
    layer(attention(4, 1, 32, 32, scale=0.6, temp=(0.3, 32)), experts(64, 8, 2, groups=(4, 2), shared=32)),
    layer(delta(3, 3, 32, 32, 4), dense(64)),
    layer(attention(2, 2, 64, 32, scale=0.4, temp=(0.2, 64)), experts(48, 6, 2, groups=(3, 2), shared=16)),
    layer(delta(4, 2, 64, 24, 3), dense(96)),
], scale=1.0, alpha=1.2, eps=1e-6))

CONFIGS = {"mixed": MIXED, "odd": ODD, "sharp": SHARP}


def middling_config(seed: int) -> dict:
    """Widths of some hundred and heads as a small real model has them: the sizes at which steps of a few hundred rows
    take the library's products, the tiled kernels and the matrix-core attention."""
    r = random.Random(seed)
    width = r.choice([256, 384, 512])
    kv = r.choice([1, 2])
    dim, vdim = r.choice([(64, 96), (128, 64), (64, 64)])
    h = r.choice([2, 4])
    layers = [
        layer(attention(kv * r.choice([2, 4]), kv, dim, vdim, temp=(0.3, r.choice([50, 128]))),
              experts(r.choice([128, 192]), 8, r.choice([1, 2, 3]), groups=(4, 2), shared=r.choice([None, 128, 64]))),
        layer(delta(2 * h, h, r.choice([64, 128]), r.choice([64, 96]), 4), dense(r.choice([320, 512]))),
        layer(delta(h, h, 48, 64, r.choice([2, 3])), experts(96, 16, 4, shared=96)),
    ]
    r.shuffle(layers)
    layers.append(again(layers, r.choice([0, 1, 2])))
    inner = {i: (r.choice([16, 24, 48]), r.choice([16, 32])) for i, e in enumerate(layers) if e["type"] == "channel_delta"}
    return dict(page_size=16, seed=seed, inner=inner, config=config(r.choice([1000, 2048]), width, layers,
                                                                    scale=r.choice([1.0, 3.0]), alpha=r.choice([1.0, 2.0])))


def random_config(seed: int) -> dict:
    """A configuration drawn from what the design allows: any order of mixers, any sizes."""
    r = random.Random(seed)
    width = r.choice([32, 48, 64, 80, 72, 100])

    def draw_mlp():
        u = r.random()
        if u < 0.2:
            return None
        if u < 0.5:
            return dense(r.choice([8, 23, 40, 72]))
        groups = r.choice([None, (1, 1), (2, 1), (2, 2), (3, 2)])
        count = (groups[0] if groups else 1) * r.choice([1, 2, 4])
        most = (groups[1] if groups else 1) * (count // (groups[0] if groups else 1))
        return experts(r.choice([8, 24, 40, 72]), count, r.randint(1, min(most, 4)), groups=groups, shared=r.choice([None, 8, 40]))

    layers, inner = [], {}
    for i in range(r.randint(2, 6)):
        if layers and r.random() < 0.2:
            layers.append(again(layers, r.choice([j for j, e in enumerate(layers) if "weights_of" not in e])))
            continue
        if r.random() < 0.5:
            kv = r.choice([1, 2, 3])
            mixer = attention(kv * r.choice([1, 2, 4]), kv, r.choice([8, 20, 32, 64]), r.choice([4, 16, 32, 40]),
                              scale=r.choice([0.1, 0.5]), temp=r.choice([None, (0.4, r.choice([1, 7, 16, 500]))]))
        else:
            kv = r.choice([1, 2, 3])
            mixer = delta(kv * r.choice([1, 2, 4]), kv, r.choice([4, 10, 16, 48, 130]), r.choice([4, 9, 16, 40]), r.choice([1, 2, 3, 4, 6]))
            inner[i] = (r.choice([1, 5, 8, 24]), r.choice([1, 6, 16, 33]))
        layers.append(layer(mixer, draw_mlp()))
    return dict(page_size=r.choice([4, 8, 16]), seed=seed, inner=inner,
                config=config(r.choice([64, 130, 300]), width, layers, scale=r.choice([0.5, 1.0, 3.0]),
                              alpha=r.choice([0.5, 1.0, 1.7, 2.5]), eps=r.choice([1e-6, 1e-5])))


def _draw(name: str, shape: tuple, seed: int, sharp: bool) -> torch.Tensor:
    g = torch.Generator().manual_seed(seed)
    n = torch.randn(shape, generator=g)
    last = name.rsplit(".", 1)[-1]
    if name.endswith("mix.norm"):
        t = 1.0 + 0.3 * n                       # a plain weight around one
    elif last in ("norm1", "norm2", "norm"):
        t = 0.3 * n                             # stored around zero
    elif last == "A_log":
        t = 0.7 * n
    elif last == "dt_bias":
        t = -3.0 + n * (2.5 if sharp else 1.5)      # decays from nearly one to well below
    elif last == "conv":
        t = 0.5 * n
    elif last == "b":
        t = n * (shape[-1] ** -0.5) * (3.0 if sharp else 1.5)
    elif last == "router":
        # logits of a few units at most: beyond some 15 a sigmoid is 1.0 in float32 and two experts tie that differ in
        # exact arithmetic
        t = n * (shape[-1] ** -0.5)
    elif last == "correction":
        t = n * (1.5 if sharp else 0.5)           # choice scores of either sign
    elif last == "sg":
        t = n * (shape[-1] ** -0.5) * 2.0
    elif name == "embed":
        t = n
    else:
        t = n * (shape[-1] ** -0.5)             # a projection keeps its input's size
    return t.to(torch.bfloat16)


def expected_shapes(c: dict) -> dict:
    """{tensor: shape} of a configuration, the inner sizes of its delta rules as `inner` has them: {layer: (decay, gate)}."""
    shapes = {n: tuple(e.shape) for n, e in build_model(copy.deepcopy(c["config"])).expected_tensors().items()}
    for i, (decay, gate) in c.get("inner", {}).items():
        p = f"l{i}.mix."
        if p + "a1" in shapes:                  # (a layer that uses another's weights has none)
            shapes[p + "a1"], shapes[p + "a2"] = (decay, shapes[p + "a1"][1]), (shapes[p + "a2"][0], decay)
            shapes[p + "g1"], shapes[p + "g2"] = (gate, shapes[p + "g1"][1]), (shapes[p + "g2"][0], gate)
    return shapes


def write_folder(name, folder: str, change=None) -> str:
    """A model folder for one of CONFIGS (or a dict of the same form): config.json and weights that make every part
    count.  `change(tensors)` may change them before they are written."""
    c = CONFIGS[name] if isinstance(name, str) else name
    tensors = {}
    for tensor_name, shape in expected_shapes(c).items():
        stable = int.from_bytes(hashlib.sha256(f"{c['seed']}:{tensor_name}".encode()).digest()[:4], "little")
        tensors[tensor_name] = _draw(tensor_name, shape, stable, bool(c.get("sharp")))
    if change is not None:
        change(tensors)
    os.makedirs(folder, exist_ok=True)
    write_safetensors(os.path.join(folder, "model.safetensors"), tensors, metadata={"format": "pt"})
    with open(os.path.join(folder, "config.json"), "w", encoding="utf-8") as f:
        json.dump(c["config"], f, indent=1, sort_keys=True)
    return folder


def requests_for(name, lengths) -> dict:
    c = CONFIGS[name] if isinstance(name, str) else name
    return {f"q{i}": random_ids(1000 * i + c["seed"], n, c["config"]["vocab"]) for i, n in enumerate(lengths)}


def plain_logits(folder: str, requests: dict, dtype=torch.float64) -> dict:
    raw, weights = read_folder(folder, dtype)
    return {rid: modasun_plain.forward(toks, weights, raw) for rid, toks in requests.items()}


def rounding_noise(folder: str, requests: dict, dtype, exact: dict) -> dict:
    """How far rounding alone carries every row: the plain implementation in float32, or in float64 with every tensor
    a bfloat16 model holds rounded to bfloat16, against the exact rows."""
    raw, weights = read_folder(folder, torch.float64)
    noise = {}
    for rid, toks in requests.items():
        if dtype == torch.float32:
            noisy = modasun_plain.forward(toks, {k: v.float() for k, v in weights.items()}, raw).double()
        else:
            noisy = modasun_plain.forward(toks, weights, raw, to_bfloat16)
        d = noisy - exact[rid]
        noise[rid] = (d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt()
    return noise


# Token 118 looks for token 119: its embedding is the other's times -1 and so are the query projections the key
# projections', so its unit query and the other's unit key have the largest product there is, whatever lies between.
SEEKER, SOUGHT = 118, 119


def seek_config(page_size: int = 16) -> dict:
    return dict(page_size=page_size, seed=54, config=config(120, 64, [
        layer(attention(2, 2, 32, 32, scale=0.6, temp=(0.1, 64)), None), layer(attention(2, 1, 32, 16, scale=0.6), dense(48))],
        scale=1.0, alpha=0.5))


def seeks(tensors: dict) -> None:
    for i in range(2):
        k = tensors[f"l{i}.mix.k"]
        tensors[f"l{i}.mix.q"] = -k.repeat(tensors[f"l{i}.mix.q"].shape[0] // k.shape[0], 1)
    tensors["embed"][SOUGHT] = -tensors["embed"][SEEKER]


def seeking(length: int, place: int) -> list:
    """A prompt whose last token seeks the one at `place`."""
    toks = [(7 * i) % SEEKER for i in range(length)]
    toks[place], toks[-1] = SOUGHT, SEEKER
    return toks
