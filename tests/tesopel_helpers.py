"""Shared by the Tesopel tests: small configurations that differ in every size and option, model folders whose
weights make every mechanism count, and the comparison with the plain implementation."""
from __future__ import annotations

import copy
import hashlib
import json
import os
import random

import torch

from duvozen_helpers import read_folder, to_bfloat16  # noqa: F401  (a folder is read the same way)
from lefisun_helpers import compare_with_rounding  # noqa: F401  (the comparison is the same)
from plain import tesopel_plain
from tokuvik_helpers import compare_rows, random_ids  # noqa: F401
from wllm_amd.parts import build_model
from wllm_amd.weights.safetensors_io import write_safetensors


def latent(heads, dim, vdim, kv_rank, window, *, scale=None, kv_from=None):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale if scale is not None else dim ** -0.5,
         "mask": {"size": window}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return "latent_attention", m


def memory(heads, dim, vdim, cap):
    return "mlstm", {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}


def retention(heads, dim, vdim, dims, base, decay):
    assert len(decay) == heads
    return "retention", {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay), "rot": {"dims": dims, "base": base}}


def layer(mixer, ff=None, limit=None):
    return {"type": mixer[0], "mixer": mixer[1], "mlp": None if ff is None else {"kind": "dense", "ff": ff, "limit": limit}}


def config(vocab, width, layers, *, logit_scale=1.0, eps=1e-6):
    return {"architecture": "Tesopel", "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_scale": logit_scale,
            "layers": layers}


# A recurrence first; a reader with a wider window than the vectors' owner, with other heads and head sizes, and one
# with a narrower window; another owner of another rank between them; a part of the head turned and the whole head;
# values narrower and wider than keys; layers without a feed-forward.
MIXED = dict(page_size=16, seed=41, config=config(160, 64, [
    layer(memory(2, 16, 32, 8.0), 96, 1.2),
    layer(latent(4, 32, 16, 80, 21, scale=0.3), 64, 3.0),
    layer(retention(2, 32, 16, 16, 10000.0, [0.8, 0.995]), 80, 0.7),
    layer(latent(2, 16, 32, 80, 50, kv_from=1)),
    layer(latent(3, 24, 24, 40, 33), 72, 2.0),
    layer(latent(1, 8, 64, 80, 7, scale=0.5, kv_from=1), 64, 5.0),
    layer(retention(3, 8, 24, 8, 50.0, [0.5, 0.9, 0.999]), 32, 1.0),
], logit_scale=0.7, eps=1e-5))

# Sizes that are no multiple of 8 (a width of 48 is one of 16), pages of 8, windows below a page and of one token, one
# head, heads of more rows than a wavefront has lanes, a window longer than every request, a rank of 9, a decay of one
# and of nothing.
ODD = dict(page_size=8, seed=42, config=config(97, 48, [
    layer(latent(3, 10, 6, 36, 5, scale=0.9), 40, 0.5),
    layer(retention(1, 130, 5, 6, 777.0, [0.97]), 56, 2.5),
    layer(latent(1, 12, 20, 9, 1, scale=0.4), 24, 1.0),
    layer(memory(3, 10, 12, 3.0), 50, 1.5),
    layer(latent(2, 6, 4, 9, 1000, kv_from=2)),
    layer(memory(1, 70, 3, 20.0)),
    layer(retention(2, 6, 9, 2, 3.0, [1.0, 0.0]), 30, 4.0),
], logit_scale=2.0, eps=1e-6))

# Attention so sharp that single keys decide, gates that open and close, limits that hold most of what they meet: a key
# lost or gained at a window's edge, a wrong page, a stale slot or a lost state moves the logits by far more than
# rounding.
SHARP = dict(page_size=16, seed=43, sharp=True, config=config(200, 96, [
    layer(latent(4, 32, 32, 64, 48, scale=0.7), 64, 0.8),
    layer(memory(3, 32, 32, 10.0), 64, 0.6),
    layer(latent(4, 16, 16, 64, 64, scale=1.0, kv_from=0), 96, 1.0),
    layer(retention(2, 32, 48, 32, 1000.0, [0.95, 0.998]), 64, 0.7),
], logit_scale=1.0, eps=1e-6))

CONFIGS = {"mixed": MIXED, "odd": ODD, "sharp": SHARP}


def reach_config(windows, page_size=16, width=64, rank=48, heads=2):
    """Latent attentions only, every one over the first one's vectors, without feed-forwards: a logit then depends on
    the tokens within the widest window and on no other."""
    layers = [layer(latent(heads, 16, 16, rank, windows[0], scale=0.5))]
    layers += [layer(latent(heads + i, 16, 24, rank, w, scale=0.4, kv_from=0)) for i, w in enumerate(windows[1:])]
    return dict(page_size=page_size, seed=44, config=config(90, width, layers))


def _decays(r, heads):
    return [round(r.choice([0.3, 0.8, 0.95, 0.99, 0.998]) + 0.001 * r.random(), 6) for _ in range(heads)]


def middling_config(seed: int) -> dict:
    """Widths of some hundred and heads as a small real model has them: the sizes at which steps of a few hundred rows
    take the library's products, the tiled kernels and the matrix-core attention."""
    r = random.Random(seed)
    width, rank = r.choice([384, 512]), r.choice([128, 160, 192])
    h = r.choice([2, 4])
    layers = [layer(latent(r.choice([4, 8]), 64, r.choice([32, 64]), rank, r.choice([90, 128, 200])), r.choice([320, 512]), 2.0),
              layer(memory(h, r.choice([64, 128]), r.choice([64, 96]), 15.0), 448, 1.0),
              layer(latent(16, 32, 32, rank, r.choice([64, 257]), kv_from=0)),
              layer(retention(h, 64, 128, r.choice([32, 64]), 10000.0, _decays(r, h)), 512, 3.0)]
    return dict(page_size=16, seed=seed, config=config(r.choice([1000, 2048]), width, layers, logit_scale=r.choice([1.0, 0.25])))


def random_config(seed: int) -> dict:
    """A configuration drawn from what the design allows: any order of mixers, any sizes."""
    r = random.Random(seed)
    width = r.choice([32, 48, 64, 80, 72, 100])
    layers, owners = [], []
    for i in range(r.randint(2, 6)):
        kind = r.choice(["latent", "memory", "retention"])
        if kind == "latent":
            source, rank = None, r.choice([8, 20, 36, 64, 96])
            if owners and r.random() < 0.5:
                source, rank = r.choice(owners)
            else:
                owners.append((i, rank))
            mixer = latent(r.choice([1, 2, 5]), r.choice([4, 16, 24]), r.choice([4, 16, 40]), rank, r.choice([1, 2, 9, 16, 31, 100]),
                           scale=r.choice([0.2, 0.7]), kv_from=source)
        elif kind == "memory":
            mixer = memory(r.choice([1, 2, 3, 6]), r.choice([4, 10, 16, 48]), r.choice([4, 16, 24, 72]), r.choice([1.0, 5.0, 15.0]))
        else:
            heads, dim = r.choice([1, 2, 3]), r.choice([4, 10, 32, 130])
            mixer = retention(heads, dim, r.choice([4, 16, 40]), r.choice([d for d in (2, 4, 10, 32) if d <= dim]),
                              r.choice([10.0, 1000.0, 1e6]), _decays(r, heads))
        ff = None if r.random() < 0.2 else r.choice([8, 24, 40, 72])
        layers.append(layer(mixer, ff, None if ff is None else r.choice([0.3, 1.0, 7.0])))
    return dict(page_size=r.choice([4, 8, 16]), seed=seed,
                config=config(r.choice([64, 130, 300]), width, layers, logit_scale=r.choice([0.3, 1.0, 2.0]), eps=r.choice([1e-6, 1e-5])))


def _draw(name: str, shape: tuple, seed: int, sharp: bool) -> torch.Tensor:
    g = torch.Generator().manual_seed(seed)
    n = torch.randn(shape, generator=g)
    last = name.rsplit(".", 1)[-1]
    if last in ("norm1", "norm2", "norm"):
        t = 1.0 + 0.3 * n                       # plain weights around one
    elif name.endswith(".f.b"):
        t = 2.5 + n * (2.0 if sharp else 1.0)     # forget gates mostly open, so that what was written long ago counts
    elif name.endswith(".i.b"):
        t = n * (2.0 if sharp else 1.0)
    elif last in ("i", "f"):
        t = n * (shape[-1] ** -0.5) * (3.0 if sharp else 1.5)
    elif name == "embed":
        t = n
    else:
        t = n * (shape[-1] ** -0.5)             # a projection keeps its input's size
    return t.to(torch.bfloat16)


def write_folder(name, folder: str) -> str:
    """A model folder for one of CONFIGS (or a dict of the same form): config.json and weights that make every part
    count."""
    c = CONFIGS[name] if isinstance(name, str) else name
    raw = copy.deepcopy(c["config"])
    tensors = {}
    for tensor_name, exp in build_model(copy.deepcopy(raw)).expected_tensors().items():
        stable = int.from_bytes(hashlib.sha256(f"{c['seed']}:{tensor_name}".encode()).digest()[:4], "little")
        tensors[tensor_name] = _draw(tensor_name, tuple(exp.shape), stable, bool(c.get("sharp")))
    os.makedirs(folder, exist_ok=True)
    write_safetensors(os.path.join(folder, "model.safetensors"), tensors, metadata={"format": "pt"})
    with open(os.path.join(folder, "config.json"), "w", encoding="utf-8") as f:
        json.dump(raw, f, indent=1, sort_keys=True)
    return folder


def requests_for(name, lengths) -> dict:
    c = CONFIGS[name] if isinstance(name, str) else name
    return {f"q{i}": random_ids(1000 * i + c["seed"], n, c["config"]["vocab"]) for i, n in enumerate(lengths)}


def plain_logits(folder: str, requests: dict, dtype=torch.float64) -> dict:
    raw, weights = read_folder(folder, dtype)
    return {rid: tesopel_plain.forward(toks, weights, raw) for rid, toks in requests.items()}


def rounding_noise(folder: str, requests: dict, dtype, exact: dict) -> dict:
    """How far rounding alone carries every row: the plain implementation in float32, or in float64 with every tensor
    a bfloat16 model holds rounded to bfloat16, against the exact rows."""
    raw, weights = read_folder(folder, torch.float64)
    noise = {}
    for rid, toks in requests.items():
        if dtype == torch.float32:
            noisy = tesopel_plain.forward(toks, {k: v.float() for k, v in weights.items()}, raw).double()
        else:
            noisy = tesopel_plain.forward(toks, weights, raw, to_bfloat16)
        d = noisy - exact[rid]
        noise[rid] = (d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt()
    return noise
