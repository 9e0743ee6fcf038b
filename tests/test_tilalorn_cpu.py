"""The Tilalorn design through the framework's host side on the CPU: configuration, tensor names, the cache plan with windows and with layers that
read another layer's keys and values, the step function under every way of cutting requests, the stream after every layer, greedy generation
through scheduler and sampler, the trace replay and the command line, with the HIP entry points replaced by the stand-ins of
``emulated_ops.py``; and that the tests' models would show a fault of every mechanism.  The kernels are tested on the GPU (``-m gpu``)."""
import json

import numpy as np
import pytest
import torch

import plain_tilalorn
import scenarios
import tiny_tilalorn
from torchlet_amd.config import TilalornConfig, ConfigError
from torchlet_amd.engine.batch import StepEntry
from torchlet_amd.engine.engine import Engine
from torchlet_amd.engine.loading import load_model, make_runner
from torchlet_amd.engine.request import Request
from torchlet_amd.registry import load_config

TOL = dict(atol=3e-4, rtol=2e-4)       # 32-bit stand-ins against a 64-bit evaluation, logits of order ten


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    root = tmp_path_factory.mktemp("tilalorn")
    return {name: tiny_tilalorn.write(name, root) for name in tiny_tilalorn.CONFIGS}


def _weights(name):
    return {k: v.double() for k, v in tiny_tilalorn.tensors_for(name).items()}


def _run(runner, steps):
    out = {}
    for s in steps:
        logits = runner.step([StepEntry(e["id"], e["tokens"], e["want"]) for e in s["entries"]])
        if logits is not None:
            out[s["step"]] = logits.numpy()
        for r in s["end"]:
            runner.release(r)
        runner.cache.check()
    return out


def test_configuration_expands_to_parts_and_names(folders):
    cfg = load_config(folders["A"])
    assert isinstance(cfg, TilalornConfig)
    spec = cfg.to_spec()
    assert [(b.kind, b.mixer.kind, b.ffn.kind if b.ffn is not None else None) for b in spec.layers] == \
        [("scaled_residual", "latent_attention", "routed_experts"), ("scaled_residual", "capped_attention", "swiglu"), ("scaled_residual", "capped_attention", None),
         ("scaled_residual", "capped_attention", "routed_experts"), ("scaled_residual", "latent_attention", "swiglu"), ("scaled_residual", "capped_attention", "swiglu")]
    assert [e.cache_of for e in spec.order] == [None, None, None, 1, None, 1] and spec.tie_head and all(b.branch_gain == 0.45 for b in spec.layers)
    lat = spec.layers[0].mixer
    assert (lat.q_rank, lat.rot_dim, lat.window, lat.gate, lat.gate_values, lat.sink, lat.kv_rank, lat.scale, lat.norm_eps) == (0, 4, 9, False, True, False, 12, 0.3, 1e-5)
    assert (lat.position.kind, lat.position.dims, lat.position.base) == ("rope_halves", 4, 40.0)
    att, reader = spec.layers[1].mixer, spec.layers[3].mixer
    assert (att.softcap, att.query_heat, att.qk_unit_norm, att.qk_norm_eps, att.qk_bias, att.v_bias, att.o_bias, att.gate, att.reads_cache, att.window) == \
        (3.0, (0.6, 6), True, 1e-5, True, True, False, True, False, None)
    assert (reader.softcap, reader.query_heat, reader.heads, reader.reads_cache, reader.v_bias) == (2.0, (0.9, 4), 3, True, False)
    moe = spec.layers[0].ffn
    assert (moe.scores, moe.choice_bias, moe.gated, moe.activation, moe.router_bias, moe.weight_scale, moe.top, moe.groups, moe.shared) == \
        ("all", False, True, "silu", False, 1.7, 2, (3, 2), None)
    assert spec.layers[1].ffn.activation == "gelu_tanh" and (spec.final_norm.kind, spec.final_norm.offset) == ("offset_rmsnorm", 1.0)
    from torchlet_amd.models.decoder import DecoderModel
    names = {n for n, s in DecoderModel(spec, torch.float32, "cpu").weight_specs().items() if not s.optional}
    assert names == set(tiny_tilalorn.tensors_for("A"))
    assert {"embed", "final.norm", "l0.norm1", "l0.mix.q", "l0.mix.dkv.norm", "l0.mix.uk", "l0.mix.g", "l0.mlp.router", "l0.mlp.e5.gate", "l1.mix.q.b", "l1.mix.k.b", "l1.mix.v.b",
            "l1.mix.g", "l1.mlp.gate", "l3.mix.q.b", "l3.mix.g", "l3.mix.o"} <= names
    assert not {"head", "l2.norm2", "l3.mix.k", "l3.mix.v", "l3.mix.k.b", "l3.mix.v.b", "l0.mlp.correction", "l1.mix.o.b", "l5.mix.k"} & names
    plain = load_config(folders["C"]).to_spec()             # no window, no cap, no temperature, no scale on the experts' weights
    assert plain.layers[1].mixer.window is None and plain.layers[0].mixer.softcap is None and plain.layers[0].mixer.query_heat is None
    assert plain.layers[0].ffn.weight_scale == 1.0 and plain.layers[3].mixer.position.dims == 4 and plain.layers[3].mixer.rot_dim == 8
    base = tiny_tilalorn.CONFIGS["A"]
    lat_layer, att_layer, _, reader_layer = base["layers"][:4]
    mixer = lambda layer, **changed: dict(layer, mixer=dict(layer["mixer"], **changed))
    moe_layer = lambda **router: dict(att_layer, mlp=dict(kind="moe", expert=dict(ff=8), router=dict(dict(experts=6, top=2), **router)))
    for bad in ([], [dict(att_layer, type="other")], [mixer(att_layer, heads=5)], [mixer(att_layer, softcap=0.0)], [mixer(att_layer, q_temp=dict(coef=0.1))],
                [mixer(att_layer, q_temp=dict(coef=0.1, every=0.5))], [mixer(lat_layer, rot=dict(dims=6, base=10.0))], [mixer(lat_layer, rot=dict(dims=3, base=10.0))],
                [mixer(lat_layer, mask=dict(size=0))], [mixer(lat_layer, kv_rank=0)], [{k: v for k, v in lat_layer.items() if k != "mixer"}],
                [reader_layer], [lat_layer, reader_layer], [att_layer, mixer(reader_layer, kv_from=0, dim=12)], [att_layer, mixer(reader_layer, kv_from=1)],
                [att_layer, mixer(reader_layer, kv_from=0), mixer(reader_layer, kv_from=1)], [moe_layer(top=7)], [moe_layer(groups=dict(count=4, keep=2))],
                [moe_layer(groups=dict(count=3, keep=4))], [moe_layer(top=3, groups=dict(count=3, keep=1))], [moe_layer(groups=dict(count=3))], [dict(att_layer, mlp=dict(kind="other"))]):
        with pytest.raises(ConfigError):
            TilalornConfig.from_dict({**base, "layers": bad})
    for bad in (dict(norm={}), dict(residual_mult="much"), dict(vocab=0)):
        with pytest.raises(ConfigError):
            TilalornConfig.from_dict({**base, **bad})


def test_cache_plan_windows_and_shared_keys(cpu_ops, folders):
    """Pages for the latent rows inside their windows and for the keys and values of the layers that have their own; a layer that reads another's gets a
    view of the same pages and may not write them."""
    _, model = load_model(folders["A"], "float32", device="cpu")
    runner = make_runner(model, page_size=4, num_pages=40, max_requests=3)
    got = [(g.need.plane_shapes, g.need.window, g.runs) for g in runner.cache.groups]
    assert got == [(((1, 16),), 9, [0]), (((3, 10), (3, 14)), None, [1]), (((1, 8), (1, 6)), None, [2]), (((1, 13),), 5, [4])]
    caches = runner.caches
    assert [c.writable for c in caches] == [True, True, True, False, True, False]
    assert all(caches[i].planes[p].data_ptr() == caches[1].planes[p].data_ptr() for i in (3, 5) for p in (0, 1))
    runner.step([StepEntry("a", list(range(30)), [])])
    held = [c - f for c, f in zip(runner.cache.capacity(), runner.cache.free_pages())]
    assert held == [3, 8, 8, 2]                      # positions 22 .. 29 and 26 .. 29 inside the windows of position 30; every position
    runner.release("a")
    assert runner.cache.free_pages() == runner.cache.capacity()
    # a mixer without keys of its own in a run that owns its cache is a mistake of the order
    from torchlet_amd.parts.base import MIXERS
    reader = MIXERS.build(model.spec.layers[3].mixer, torch.float32, torch.device("cpu"))
    with pytest.raises(ValueError):
        reader.mix(torch.zeros(1, reader.in_width), torch.zeros(1, 40), None, caches[1], torch.zeros(1, reader.mix_width))


FAULTS = {
    "a window one token wider": ("mask_matrix", lambda f: lambda T, window, dtype=torch.float64: f(T, window + 1 if window else window, dtype)),
    "a window one token narrower": ("mask_matrix", lambda f: lambda T, window, dtype=torch.float64: f(T, max(1, window - 1) if window else window, dtype)),
    "no window": ("mask_matrix", lambda f: lambda T, window, dtype=torch.float64: f(T, None, dtype)),
    "angles from the next position": ("rotate_halves", lambda f: lambda x, p, dims, base: f(x, p + 1 if x.dim() == 3 else p, dims, base)),
    "a temperature one position late": ("query_temperature", lambda f: lambda p, coef, every, dtype=torch.float64: f(p - 1, coef, every, dtype)),
    "no temperature": ("query_temperature", lambda f: lambda p, coef, every, dtype=torch.float64: torch.ones(len(p), dtype=dtype)),
    "no cap": ("soft_cap", lambda f: lambda s, cap: s),
    "gelu by the error function": ("gelu_tanh", lambda f: torch.nn.functional.gelu),
    "no groups": ("grouped_router", lambda f: lambda h, w, router, gaps=None: f(h, w, {k: v for k, v in router.items() if k != "groups"}, gaps)),
    "weights renormalised": ("grouped_router", lambda f: lambda h, w, router, gaps=None: (lambda c, s: (c, s / s.sum(-1, keepdim=True)))(*f(h, w, router, gaps))),
}


@pytest.mark.parametrize("fault", FAULTS)
def test_models_of_the_tests_show_every_fault(monkeypatch, fault):
    """The plain implementation with one mechanism changed gives logits that differ by far more than the tests' bounds, in configuration A or B."""
    worst = 0.0
    for name in ("A", "B"):
        w = _weights(name)
        g = torch.Generator().manual_seed(4)
        ids = torch.randint(0, tiny_tilalorn.CONFIGS[name]["vocab"], (60,), generator=g).tolist()
        want = plain_tilalorn.forward(tiny_tilalorn.CONFIGS[name], w, ids)[0]
        where, change = FAULTS[fault]
        with monkeypatch.context() as m:
            m.setattr(plain_tilalorn, where, change(getattr(plain_tilalorn, where)))
            got = plain_tilalorn.forward(tiny_tilalorn.CONFIGS[name], w, ids)[0]
        worst = max(worst, float((got - want).abs().max()))
    assert worst > (5 if fault == "gelu by the error function" else 200) * TOL["atol"], worst


@pytest.mark.parametrize("name", ["A", "B", "C"])
@pytest.mark.parametrize("mode", ["whole", "tail_singles", "portions", "mixed"])
def test_step_function_equals_plain_under_every_split(cpu_ops, folders, name, mode):
    lengths = [37, 5, 50, 1, 18, 33] if name != "B" else [75, 1, 27]
    seqs, refs = tiny_tilalorn.sequences(name, _weights(name), lengths)
    steps = scenarios.number(getattr(scenarios, mode)(seqs) if mode != "tail_singles" else scenarios.tail_singles(seqs, tail=9))
    page = tiny_tilalorn.PAGE_SIZES[name]
    _, model = load_model(folders[name], "float32", device="cpu")
    runner = make_runner(model, page_size=page, num_pages=-(-scenarios.max_tokens_needed(steps, unit=page) // page) + 1, max_requests=4)
    scenarios.check(steps, _run(runner, steps), refs, TOL, f"{name}/{mode}")
    assert runner.cache.live_requests() == [] and runner.cache.free_pages() == runner.cache.capacity()


@pytest.mark.parametrize("seed", range(4))
def test_configurations_drawn_at_random(cpu_ops, tmp_path, seed):
    """Layers of any kind in any order, through the host side: portions and mixed batches against plain."""
    import random
    rnd = random.Random(900 + seed)
    conf = tiny_tilalorn.random_config(rnd, big=False)
    page = rnd.choice([4, 8, 16])
    folder = tiny_tilalorn.write(f"random{seed}", tmp_path, config=conf, seed=seed)
    w = {k: v.double() for k, v in tiny_tilalorn.tensors_for("", 1.0, conf, seed).items()}
    seqs, refs = tiny_tilalorn.sequences("", w, [rnd.randint(1, 60) for _ in range(4)], seed=seed, config=conf, min_gap=1e-3)
    _, model = load_model(folder, "float32", device="cpu")
    for mode in ("portions", "mixed"):
        steps = scenarios.number(getattr(scenarios, mode)(seqs))
        runner = make_runner(model, page_size=page, num_pages=-(-scenarios.max_tokens_needed(steps, unit=page) // page) + 1, max_requests=4)
        scenarios.check(steps, _run(runner, steps), refs, TOL, f"{conf}/{mode}")
        assert runner.cache.free_pages() == runner.cache.capacity()


def test_stream_after_every_layer_against_plain(cpu_ops, folders):
    ids = [5, 17, 3, 60, 2, 2, 41, 9, 30, 11, 90, 4, 4, 8]
    _, want = plain_tilalorn.forward(tiny_tilalorn.CONFIGS["A"], _weights("A"), ids)
    _, model = load_model(folders["A"], "float32", device="cpu")
    runner = make_runner(model, page_size=4, num_pages=12, max_requests=1)
    seen = []
    import emulated_ops

    def settled(stream):            # what the next norm would see: the pending output added times its factor
        x = stream.residual.clone()
        emulated_ops.sandwich_norm(x, stream.pending, None, 0.0, None, torch.ones(1), 1e-5, torch.empty_like(x), branch_gain=stream.gain)
        return x

    for block in model.blocks:
        inner = block.forward
        block.forward = lambda stream, ctx, cache, inner=inner: (lambda s: (seen.append(settled(s)), s)[1])(inner(stream, ctx, cache))
    runner.step([StepEntry("a", ids, [len(ids) - 1])])
    assert len(seen) == 6
    for got, ref in zip(seen, want):
        torch.testing.assert_close(got.double(), ref, atol=5e-5, rtol=1e-5)


def _greedy(cfg, w, prompt, n):
    ids = list(prompt)
    for _ in range(n):
        ids.append(int(plain_tilalorn.forward(cfg, w, ids)[0][-1].argmax()))
    return ids[len(prompt):]


def test_greedy_generation_through_scheduler_and_sampler(cpu_ops, folders):
    """Prompts in portions of at most 12 tokens beside decode tokens, five requests over three slots (slots and pages are used again),
    steps enqueued ahead of their tokens, against the plain loop."""
    w = _weights("B")
    cfg = tiny_tilalorn.CONFIGS["B"]
    g = torch.Generator().manual_seed(11)
    prompts = [torch.randint(0, cfg["vocab"], (n,), generator=g).tolist() for n in (5, 17, 45, 1, 9)]
    _, model = load_model(folders["B"], "float32", device="cpu")
    engine = Engine(make_runner(model, page_size=16, num_pages=14, max_requests=3), max_tokens_per_step=12)
    reqs = [Request(prompt_tokens=p, seed=i, max_new_tokens=6) for i, p in enumerate(prompts)]
    for r in reqs:
        engine.add_request(r)
    engine.run_until_done()
    for r, p in zip(reqs, prompts):
        assert r.output_tokens == _greedy(cfg, w, p, 6)
    assert engine.runner.cache.live_requests() == [] and len({tuple(r.output_tokens) for r in reqs}) > 1


def test_trace_replay_reads_the_architecture_from_the_folder(cpu_ops, folders, tmp_path, monkeypatch):
    from torchlet_amd.engine import loading, trace
    monkeypatch.setattr(loading, "require_gpu", lambda: torch.device("cpu"))
    seqs, refs = tiny_tilalorn.sequences("A", _weights("A"), [13, 6, 40])
    steps = scenarios.number(scenarios.mixed(seqs, seed=1))
    args = trace.parse_args(["--model", str(folders["A"]), "--dtype", "float32", "--out", str(tmp_path / "out"),
                             "--max-tokens", str(scenarios.max_tokens_needed(steps)), "--page-size", "4"])
    import io
    said = io.StringIO()
    assert trace.run(args, [json.dumps(s) for s in steps], out=said) == 0
    assert said.getvalue().split() == [w for s in steps for w in ("done", str(s["step"]))]
    out = {s["step"]: np.fromfile(tmp_path / "out" / f"{s['step']}.f32", dtype="<f4").reshape(-1, 97) for s in steps
           if any(e["want"] for e in s["entries"])}
    scenarios.check(steps, out, refs, TOL, "trace replay")


def test_command_line_writes_a_random_folder_of_the_architecture(cpu_ops, tmp_path):
    from safetensors import safe_open
    from torchlet_amd.llm import main
    from torchlet_amd.models.decoder import DecoderModel
    src = tmp_path / "config.json"
    src.write_text(json.dumps(tiny_tilalorn.CONFIGS["A"]))
    assert main(["init", "--config", str(src), "--seed", "3", "--out", str(tmp_path / "out")]) == 0
    cfg = load_config(tmp_path / "out")
    assert isinstance(cfg, TilalornConfig) and cfg.layers == tiny_tilalorn.CONFIGS["A"]["layers"]
    with safe_open(str(tmp_path / "out" / "model.safetensors"), framework="pt") as f:
        stored = set(f.keys())
    assert stored == {n for n, s in DecoderModel(cfg.to_spec(), torch.float32, "cpu").weight_specs().items() if not s.optional}
    _, model = load_model(tmp_path / "out", "float32", device="cpu")
    logits = make_runner(model, page_size=4, num_pages=8, max_requests=1).step([StepEntry("a", [1, 2, 3, 4, 5], [4])])
    assert logits.shape == (1, 97) and bool(torch.isfinite(logits).all())
