"""Tiny random-weight folders of the Tilalorn design for the tests: sizes chosen so that what could coincide does not (plain against rotated
query/key dimensions against value size against latent, heads against key heads, window against page, steps of the query's temperature against
pages, experts against groups), every kind of layer in several orders, layers that read an earlier layer's keys and values (one source for
several layers, a source that is not the layer just before), layers without a feed-forward, routers with one group, as many groups as experts,
one kept group, all kept, one choice, as many choices as the kept groups hold, at sizes that the matrix-core kernels take and at sizes they
leave to the general ones."""
import json
from pathlib import Path

import torch
from safetensors.torch import save_file


def _latent(heads, dim, rot_dim, vdim, kv_rank, scale, base, window=None, dims=None):
    m = dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, scale=scale, rot=dict(dims=dims or rot_dim, base=base))
    if window is not None:
        m["mask"] = dict(size=window)
    return m


def _attention(heads, kv_heads, dim, vdim, scale, softcap=None, temp=None, kv_from=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale)
    if softcap is not None:
        m["softcap"] = softcap
    if temp is not None:
        m["q_temp"] = dict(coef=temp[0], every=temp[1])
    if kv_from is not None:
        m["kv_from"] = kv_from
    return m


def _dense(ff):
    return dict(kind="dense", ff=ff)


def _moe(ff, experts, top, groups=None, scale=None):
    m = dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, top=top))
    if groups is not None:
        m["router"]["groups"] = dict(count=groups[0], keep=groups[1])
    if scale is not None:
        m["router"]["scale"] = scale
    return m


CONFIGS = {
    # nothing coincides and nothing is a multiple of a tile; pages of 4; windows of 9 and 5; a temperature that moves every 6 positions; layer 3
    # and layer 5 read layer 1's keys and values, past a layer with its own; a layer without a feed-forward
    "A": dict(architecture="Tilalorn", vocab=97, width=40, norm=dict(eps=1e-5), residual_mult=0.45, layers=[
        dict(type="latent_attention", mixer=_latent(3, 6, 4, 10, 12, 0.3, 40.0, window=9), mlp=_moe(12, 6, 2, (3, 2), 1.7)),
        dict(type="attention", mixer=_attention(6, 3, 10, 14, 0.35, softcap=3.0, temp=(0.6, 6)), mlp=_dense(24)),
        dict(type="attention", mixer=_attention(2, 1, 8, 6, 0.4, softcap=7.0, temp=(0.3, 11)), mlp=None),
        dict(type="attention", mixer=_attention(3, 3, 10, 14, 0.5, softcap=2.0, temp=(0.9, 4), kv_from=1), mlp=_moe(8, 8, 3, (4, 2), 0.8)),
        dict(type="latent_attention", mixer=_latent(5, 4, 6, 3, 7, 0.4, 900.0, window=5), mlp=_dense(20)),
        dict(type="attention", mixer=_attention(6, 3, 10, 14, 0.25, softcap=5.0, temp=(0.5, 9), kv_from=1), mlp=_dense(28)),
    ]),
    # sizes of the matrix-core kernels, pages of 16; windows that are no multiples of the page; a latent that does not split evenly over waves
    "B": dict(architecture="Tilalorn", vocab=80, width=64, norm=dict(eps=3e-6), residual_mult=0.35, layers=[
        dict(type="attention", mixer=_attention(4, 2, 64, 48, 0.12, softcap=8.0, temp=(0.5, 32)), mlp=_moe(32, 8, 3, (4, 2), 2.2)),
        dict(type="latent_attention", mixer=_latent(4, 32, 16, 48, 80, 0.18, 50000.0, window=40), mlp=_dense(96)),
        dict(type="attention", mixer=_attention(8, 2, 64, 48, 0.15, softcap=12.0, temp=(0.25, 48), kv_from=0), mlp=_dense(64)),
        dict(type="latent_attention", mixer=_latent(2, 64, 32, 32, 128, 0.1, 10000.0, window=21), mlp=None),
    ]),
    # what another model may make equal or one: no window, a window of one token, one head, no cap, no temperature and one that moves at every
    # position, a rotation over a part of the rotated numbers, one group and as many groups as experts, one kept, one expert per token and as
    # many as the kept groups hold, a factor of one on the branches
    "C": dict(architecture="Tilalorn", vocab=53, width=36, norm=dict(eps=2e-5), residual_mult=1.0, layers=[
        dict(type="attention", mixer=_attention(1, 1, 12, 12, 0.3), mlp=_moe(10, 3, 1, (1, 1))),
        dict(type="latent_attention", mixer=_latent(1, 16, 2, 16, 16, 0.25, 100.0), mlp=_dense(36)),
        dict(type="attention", mixer=_attention(3, 1, 12, 12, 0.45, softcap=4.0, temp=(0.2, 1), kv_from=0), mlp=_moe(6, 4, 2, (4, 2), 1.0)),
        dict(type="latent_attention", mixer=_latent(5, 4, 8, 2, 6, 0.5, 50.0, window=1, dims=4), mlp=_moe(6, 6, 2, (3, 1))),
    ]),
}
SEEDS = {"A": 61, "B": 62, "C": 63}
PAGE_SIZES = {"A": 4, "B": 16, "C": 8}


def tensors_for(name: str, sharpen: float = 1.0, config: dict | None = None, seed: int | None = None) -> dict[str, torch.Tensor]:
    """bfloat16 tensors of configuration ``name`` (or of ``config``): the framework's random draw, then matrices scaled up to give activations of
    order one, and norm weights and biases away from the trivial ones.  ``sharpen`` multiplies the query projections (of the latent attentions; an
    attention's queries are normed).  Clear choices of experts: every token's embedding carries the layer's experts' directions of the stream in
    an order of its own, expert e's router row looks along direction e, and what the sublayers write into the stream is kept off those
    directions, so that no choice hangs on the last bits of a score, where a reduced-precision engine would be free to choose otherwise."""
    from torchlet_amd.registry import config_class
    from torchlet_amd.weights.random_init import random_tensors
    conf = config or CONFIGS[name]
    seed = SEEDS[name] if seed is None else seed
    cfg = config_class("Tilalorn").from_dict(conf)
    g = torch.Generator().manual_seed(seed + 100)
    width, vocab = conf["width"], conf["vocab"]
    routed = {n: layer["mlp"]["router"]["experts"] for n, layer in enumerate(conf["layers"]) if layer.get("mlp") and layer["mlp"]["kind"] == "moe"}
    basis = torch.linalg.qr(torch.randn(width, max(1, min(width // 2, sum(routed.values()))), generator=g)).Q.T * width ** 0.5
    directions, code, at = {}, torch.zeros(vocab, width), 0
    for n, experts in routed.items():
        directions[n] = basis[[(at + e) % basis.shape[0] for e in range(experts)]]
        at += experts
        for t in range(vocab):           # every token ranks the layer's experts, in steps that rounding cannot turn round
            rank = torch.randperm(experts, generator=g)
            code[t] += (torch.linspace(1.0, -1.0, experts)[:, None] * directions[n][rank]).sum(0)
    drawn = random_tensors(cfg, seed, torch.float32)
    norms = {k: (torch.randn(v.shape, generator=g) * 0.3).to(torch.bfloat16).float() for k, v in drawn.items()
             if k.rsplit(".", 1)[-1] in ("norm1", "norm2") or k == "final.norm"}
    out = {}
    for k, v in drawn.items():
        leaf, layer = k.rsplit(".", 1)[-1], k.split(".")[0]
        if k in norms:
            out[k] = norms[k].to(torch.bfloat16)
            continue
        if v.dim() == 2 and k != "embed":
            v = v * (50.0 / v.shape[1] ** 0.5)                  # N(0, 1 / fan_in)
        if k == "embed":
            v = v * 8.0 + 0.4 * code
        if leaf in ("o", "down"):
            v = v * 2.0
            if routed:                                          # the sublayers' outputs stay off the routers' directions
                v = v - basis.T @ (basis @ v) / width
        if leaf == "router":
            v = v * 0.02 + directions[int(layer[1:])] * (5.0 / width) / (1.0 + norms[f"{layer}.norm2"])
        if leaf == "q" and ".mix." in k:
            v = v * sharpen
        if leaf == "b":
            v = torch.randn(v.shape, generator=g) * 0.4
        if k.endswith(".dkv.norm"):
            v = 1.0 + (v - 1.0) * 8.0
        out[k] = v.to(torch.bfloat16)
    return out


def write(name: str, root: Path, dtype=torch.bfloat16, sharpen: float = 1.0, config: dict | None = None, seed: int | None = None) -> Path:
    folder = Path(root) / f"tilalorn_{name}"
    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(config or CONFIGS[name], indent=1))
    save_file({k: v.to(dtype).contiguous() for k, v in tensors_for(name, sharpen, config, seed).items()}, str(folder / "model.safetensors"))
    return folder


def sequences(name: str, weights, lengths, seed: int = 0, config: dict | None = None, min_gap: float = 0.06):
    """Token sequences of the given lengths for which no token's choice (of a group, of an expert) leads what it leaves out by less than
    ``min_gap`` in the logarithm of the score, with the plain logits of each."""
    import plain_tilalorn
    cfg = config or CONFIGS[name]
    smallest = []
    for s in range(seed, seed + 40):
        g = torch.Generator().manual_seed(s)
        seqs = {f"r{i}": torch.randint(0, cfg["vocab"], (n,), generator=g).tolist() for i, n in enumerate(lengths)}
        gaps: list[float] = []
        refs = {r: plain_tilalorn.forward(cfg, weights, t, gaps=gaps)[0] for r, t in seqs.items()}
        if not gaps or min(gaps) > min_gap:
            return seqs, refs
        smallest.append(min(gaps))
    raise AssertionError(f"no seed gives every token a clear choice of experts (smallest margins up to {max(smallest):.4f})")


def random_config(rnd, big: bool) -> dict:
    """A configuration drawn at random: one to six layers of either kind in any order, sizes of the matrix-core kernels (``big``) or small odd
    ones, windows from one token up, attention layers that read an earlier one's keys and values where there is one, with or without caps,
    temperatures, groups and feed-forwards."""
    layers: list[dict] = []
    for _ in range(rnd.randint(1, 6)):
        if rnd.random() < 0.45:
            kind = "latent_attention"
            rank, rot = rnd.choice([(64, 32), (80, 16), (112, 16), (256, 64), (160, 32)] if big else [(5, 2), (12, 6), (24, 4)])
            mixer = _latent(rnd.choice([1, 2, 4, 5]), rnd.choice([32, 64] if big else [4, 6, 10]), rot, rnd.choice([16, 32, 80] if big else [3, 8, 12]),
                            rank, rnd.choice([0.1, 0.25]), rnd.choice([100.0, 10000.0, 1e6]), rnd.choice([None, 1, 3, 7, 16, 33, 50]))
        else:
            kind = "attention"
            sources = [i for i, other in enumerate(layers) if other["type"] == "attention" and "kv_from" not in other["mixer"]]
            source = rnd.choice(sources) if sources and rnd.random() < 0.5 else None
            shape = layers[source]["mixer"] if source is not None else dict(kv_heads=rnd.choice([1, 2, 3]), dim=rnd.choice([32, 64, 96, 128] if big else [4, 6, 10, 24]),
                                                                              vdim=rnd.choice([16, 48, 64, 112] if big else [3, 8, 12]))
            mixer = _attention(shape["kv_heads"] * rnd.choice([1, 2, 4]), shape["kv_heads"], shape["dim"], shape["vdim"], rnd.choice([0.1, 0.25, shape["dim"] ** -0.5]),
                               rnd.choice([None, 1.5, 20.0]), rnd.choice([None, (0.5, 1), (0.3, 7), (1.0, 64)]), source)
        roll = rnd.random()
        if roll < 0.15:
            mlp = None
        elif roll < 0.55:
            mlp = _dense(rnd.choice([16, 48, 72]))
        else:
            experts = rnd.choice([2, 4, 6])
            count = rnd.choice([n for n in (1, 2, 3, experts) if experts % n == 0])
            keep = rnd.randint(1, count)
            mlp = _moe(rnd.choice([8, 24, 32]), experts, rnd.randint(1, min(3, keep * experts // count)), rnd.choice([None, (count, keep)]) if keep == count else (count, keep),
                       rnd.choice([None, 1.0, 2.2]))
        layers.append(dict(type=kind, mixer=mixer, mlp=mlp))
    return dict(architecture="Tilalorn", vocab=rnd.choice([31, 90, 300]), width=rnd.choice([64, 128] if big else [24, 40, 56]),
                norm=dict(eps=rnd.choice([1e-5, 1e-6, 3e-4])), residual_mult=rnd.choice([1.0, 0.25, 0.55]), layers=layers)
