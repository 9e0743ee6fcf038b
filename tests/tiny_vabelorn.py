"""Tiny random-weight folders of the Vabelorn design for the tests: sizes chosen so that what could coincide does not (key size against value
size against rotated dimensions, heads against key heads, decay rank against token-input size), both kinds of layer in several orders, layers
with and without a feed-forward, YaRN scaling whose ramp lies inside, before and behind the pairs, none, sizes that the matrix-core kernels
take and sizes they leave to the general ones."""
import json
from pathlib import Path

import torch
from safetensors.torch import save_file


def _wkv(heads, dim, rank):
    return dict(heads=heads, dim=dim, decay_rank=rank)


def _attention(heads, kv_heads, dim, vdim, scale, rot=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale)
    if rot is not None:
        m["rot"] = rot
    return m


def _rot(dims, base, scaling=None):
    r = dict(dims=dims, base=base)
    if scaling is not None:
        r["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return r


def _dense(ff):
    return dict(kind="dense", ff=ff)


CONFIGS = {
    # nothing coincides and nothing is a multiple of a tile or of four; pages of 4
    "A": dict(architecture="Vabelorn", vocab=97, width=42, norm=dict(eps=1e-5), logit_scale=0.6, token_side=dict(dim=5), layers=[
        dict(type="attention", mixer=_attention(6, 2, 10, 14, 0.4, _rot(6, 50.0, (3.0, 40, 4.0, 0.5))), mlp=_dense(26)),
        dict(type="wkv", mixer=_wkv(3, 7, 5), mlp=_dense(19)),
        dict(type="wkv", mixer=_wkv(2, 11, 9), mlp=None),
        dict(type="attention", mixer=_attention(4, 4, 8, 6, 0.5, _rot(8, 900.0)), mlp=None),
    ]),
    # sizes of the matrix-core kernels, pages of 16
    "B": dict(architecture="Vabelorn", vocab=80, width=64, norm=dict(eps=3e-6), logit_scale=0.5, token_side=dict(dim=16), layers=[
        dict(type="wkv", mixer=_wkv(3, 32, 16), mlp=None),
        dict(type="attention", mixer=_attention(4, 2, 64, 32, 0.125, _rot(32, 20000.0, (8.0, 128, 16.0, 1.0))), mlp=_dense(96)),
        dict(type="wkv", mixer=_wkv(1, 64, 24), mlp=_dense(64)),
        dict(type="attention", mixer=_attention(2, 1, 32, 96, 0.2, _rot(16, 100.0, (2.0, 4096, 64.0, 2.0))), mlp=_dense(32)),
    ]),
    # what another model may make equal or one: one head everywhere, one key, value and rotated size, no scaling, a token input and a decay
    # rank of one, a factor of one on the logits, a scaling factor of one
    "C": dict(architecture="Vabelorn", vocab=53, width=36, norm=dict(eps=2e-4), logit_scale=1.0, token_side=dict(dim=1), layers=[
        dict(type="attention", mixer=_attention(1, 1, 12, 12, 0.3, _rot(12, 60.0)), mlp=_dense(36)),
        dict(type="attention", mixer=_attention(3, 3, 4, 2, 0.6, _rot(2, 7.0, (1.0, 16, 2.0, 1.0))), mlp=None),
        dict(type="wkv", mixer=_wkv(1, 1, 1), mlp=_dense(12)),
        dict(type="wkv", mixer=_wkv(1, 36, 4), mlp=None),
    ]),
}
SEEDS = {"A": 43, "B": 44, "C": 46}
PAGE_SIZES = {"A": 4, "B": 16, "C": 8}


def tensors_for(name: str, sharpen: float = 1.0, config: dict | None = None, seed: int | None = None, remember: bool = False) -> dict[str, torch.Tensor]:
    """bfloat16 tensors of configuration ``name`` (or of ``config``): the framework's random draw, then matrices scaled up to give activations
    of order one, and norm weights and bonuses away from the trivial ones.  ``sharpen`` multiplies the queries' norm weights (the scores).
    ``remember``: decays close to one (a state keeps hundreds of tokens)."""
    from torchlet_amd.registry import config_class
    from torchlet_amd.weights.random_init import random_tensors
    conf = config or CONFIGS[name]
    seed = SEEDS[name] if seed is None else seed
    cfg = config_class("Vabelorn").from_dict(conf)
    g = torch.Generator().manual_seed(seed + 100)
    out = {}
    for k, v in random_tensors(cfg, seed, torch.float32).items():
        leaf = k.rsplit(".", 1)[-1]
        if k in ("embed", "side.embed"):
            v = v * 50.0
        elif k.endswith(".u"):
            v = torch.randn(v.shape, generator=g) * 0.7
        elif leaf == "w0":
            v = v if not remember else v * 0.2 - 7.0
        elif v.dim() == 2:
            v = v * (50.0 / v.shape[1] ** 0.5)                  # N(0, 1 / fan_in)
            if leaf in ("w1", "w2") and remember:
                v = v * 0.2
        elif leaf in ("norm", "norm1", "norm2"):
            v = 1.0 + torch.randn(v.shape, generator=g) * 0.3
        if k.endswith(".q.norm"):
            v = v * sharpen
        out[k] = v.to(torch.bfloat16)
    return out


def write(name: str, root: Path, dtype=torch.bfloat16, config: dict | None = None, tensors: dict | None = None) -> Path:
    """A folder whose ``config.json`` does not say the decays' ranks: the tensors do."""
    folder = Path(root) / f"vabelorn_{name}"
    folder.mkdir(parents=True, exist_ok=True)
    conf = json.loads(json.dumps(config or CONFIGS[name]))
    tensors = tensors_for(name) if tensors is None else tensors
    for layer in conf["layers"]:
        layer["mixer"].pop("decay_rank", None)
    (folder / "config.json").write_text(json.dumps(conf, indent=1))
    save_file({k: v.to(dtype).contiguous() for k, v in tensors.items()}, str(folder / "model.safetensors"))
    return folder


def sequences(weights, lengths, config: dict, seed: int = 0):
    """Token sequences of the given lengths with the plain logits of each."""
    import plain_vabelorn
    g = torch.Generator().manual_seed(seed)
    seqs = {f"r{i}": torch.randint(0, config["vocab"], (n,), generator=g).tolist() for i, n in enumerate(lengths)}
    return seqs, {r: plain_vabelorn.forward(config, weights, t)[0] for r, t in seqs.items()}


def random_config(rnd, big: bool) -> dict:
    """A configuration drawn at random: one to five layers of either kind in any order, sizes of the matrix-core kernels (``big``) or small odd
    ones, with or without scaling and feed-forwards."""
    layers = []
    for _ in range(rnd.randint(1, 5)):
        if rnd.random() < 0.5:
            mixer, kind = _wkv(rnd.choice([1, 2, 3, 5]), rnd.choice([32, 64, 96, 130] if big else [3, 8, 13, 20]), rnd.choice([1, 4, 7, 32])), "wkv"
        else:
            dim = rnd.choice([32, 64, 96, 128] if big else [4, 6, 10, 24])
            kv_heads = rnd.choice([1, 2, 3])
            scaling = rnd.choice([None, (4.0, 64, 32.0, 1.0), (2.0, 1000, 8.0, 0.5), (16.0, 8, 2.0, 1.0), (6.0, 300, 3.0, 3.0)])
            rot = _rot(rnd.choice([d for d in (2, 4, 8, 16, 32, 64, 128) if d <= dim]), rnd.choice([20.0, 10000.0, 1e6]), scaling)
            mixer = _attention(kv_heads * rnd.choice([1, 2, 4]), kv_heads, dim, rnd.choice([16, 32, 64, 96] if big else [2, 6, 8, 12]),
                               rnd.choice([0.1, 0.25, dim ** -0.5]), rot)
            kind = "attention"
        layers.append(dict(type=kind, mixer=mixer, mlp=None if rnd.random() < 0.4 else _dense(rnd.choice([16, 48, 72, 23]))))
    return dict(architecture="Vabelorn", vocab=rnd.choice([31, 90, 300]), width=rnd.choice([64, 128] if big else [24, 39, 56]),
                norm=dict(eps=rnd.choice([1e-5, 1e-6, 3e-4])), logit_scale=rnd.choice([1.0, 0.25, 0.7]) * 0.2, token_side=dict(dim=rnd.choice([1, 3, 8, 24])),
                layers=layers)
