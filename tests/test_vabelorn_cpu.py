"""The Vabelorn design through the framework's host side on the CPU: configuration, tensor names and sizes that only the tensors say, the
cache plan, rotation frequencies, the step function under every way of cutting requests, the stream after every layer, greedy generation
through scheduler and sampler, the trace replay and the command line, with the HIP entry points replaced by the stand-ins of
``emulated_ops.py``; and the plain implementation against itself.  The kernels are tested on the GPU (``-m gpu``)."""
import io
import json
import math

import numpy as np
import pytest
import torch

import plain_vabelorn
import scenarios
import tiny_vabelorn
from torchlet_amd.config import ConfigError, HalfRotarySpec, PairRotarySpec, VabelornConfig
from torchlet_amd.engine.batch import StepEntry
from torchlet_amd.engine.engine import Engine
from torchlet_amd.engine.loading import load_model, make_runner
from torchlet_amd.engine.request import Request
from torchlet_amd.parts import POSITION_ENCODINGS
from torchlet_amd.registry import load_config
from torchlet_amd.weights.loader import WeightError

TOL = dict(atol=3e-4, rtol=2e-4)       # 32-bit stand-ins against a 64-bit evaluation, logits of order one to four


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    root = tmp_path_factory.mktemp("vabelorn")
    return {name: tiny_vabelorn.write(name, root) for name in tiny_vabelorn.CONFIGS}


def _weights(name):
    return {k: v.double() for k, v in tiny_vabelorn.tensors_for(name).items()}


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
    assert isinstance(cfg, VabelornConfig)
    spec = cfg.to_spec()
    assert [(b.kind, b.mixer.kind, b.ffn.kind if b.ffn is not None else None, b.side.dim) for b in spec.layers] == \
        [("output_norm_residual", "capped_attention", "swiglu", 5), ("output_norm_residual", "wkv", "swiglu", 5),
         ("output_norm_residual", "wkv", None, 5), ("output_norm_residual", "capped_attention", None, 5)]
    att = spec.layers[0].mixer
    assert (att.heads, att.kv_heads, att.dim, att.vdim, att.scale, att.qk_norm, att.qk_norm_eps, att.fixed_sink, att.sink, att.value_norm) == \
        (6, 2, 10, 14, 0.4, True, 1e-5, 0.0, False, True)
    assert (att.position.kind, att.position.dims, att.position.base, att.position.yarn) == ("rope_pairs", 6, 50.0, (3.0, 40.0, 4.0, 0.5))
    assert (att.value_position.dims, att.value_position.base, att.value_position.yarn) == (14, 50.0, None)
    assert spec.layers[3].mixer.position.yarn is None
    wkv = spec.layers[1].mixer
    assert (wkv.heads, wkv.dim, wkv.vdim, wkv.norm_eps) == (3, 7, 7, 1e-5)
    assert spec.layers[0].ffn.activation == "silu" and spec.tie_head and spec.logit_scale == 0.6 and spec.embed_scale == 1.0
    assert (spec.token_side.name, spec.token_side.dim) == ("side.embed", 5) and (spec.final_norm.offset, spec.final_norm.gain) == (0.0, 1.0)
    from torchlet_amd.models.decoder import DecoderModel
    names = {n for n, s in DecoderModel(spec, torch.float32, "cpu").weight_specs().items() if not s.optional}
    assert names == set(tiny_vabelorn.tensors_for("A"))
    assert {"embed", "side.embed", "final.norm", "l0.norm1", "l0.norm2", "l0.mix.q.norm", "l0.side.gate", "l1.mix.mu.w", "l1.mix.w0", "l1.mix.u",
            "l2.side.norm", "l1.mlp.down"} <= names
    assert not {"l2.norm2", "l3.norm2", "l0.mix.sink", "head"} & names
    base = tiny_vabelorn.CONFIGS["A"]
    att_layer, wkv_layer = base["layers"][0], base["layers"][1]
    mix = lambda **kw: dict(layers=[dict(att_layer, mixer=dict(att_layer["mixer"], **kw))])
    for bad in (dict(layers=[]), dict(layers=[dict(att_layer, type="other")]), dict(norm={}), dict(logit_scale="much"), dict(token_side=dict(dim=0)),
                mix(heads=5), mix(vdim=7), mix(rot=dict(dims=12, base=10.0)), mix(rot=dict(dims=5, base=10.0)), mix(rot=dict(dims=6)),
                mix(rot=dict(dims=6, base=10.0, scaling=dict(factor=2.0))), mix(rot=dict(dims=6, base=10.0, scaling=dict(factor=2.0, original=9, fast=0, slow=1))),
                dict(layers=[dict(wkv_layer, mixer=dict(heads=2))]), dict(layers=[dict(att_layer, mlp=dict(kind="moe"))])):
        with pytest.raises(ConfigError):
            VabelornConfig.from_dict({**base, **bad})


def test_sizes_that_only_the_tensors_say(folders, tmp_path):
    """The decay's inner size is not in config.json: each layer takes its tensors' own; tensors that disagree, or another size that does not
    fit, are refused."""
    _, model = load_model(folders["A"], "float32", device="cpu")
    assert [tuple(model.blocks[i].mixer.w1.shape) for i in (1, 2)] == [(5, 42), (9, 42)] and tuple(model.blocks[2].mixer.w2t.shape) == (9, 22)
    good = tiny_vabelorn.tensors_for("A")
    bad = dict(good, **{"l1.mix.w1": good["l1.mix.w1"][:4]})
    with pytest.raises(ConfigError, match="inner sizes"):
        load_model(tiny_vabelorn.write("bad", tmp_path, config=tiny_vabelorn.CONFIGS["A"], tensors=bad), "float32", device="cpu")
    bad = dict(good, **{"l1.mix.w2": good["l1.mix.w2"][:-1], "side.embed": good["side.embed"][:, :-1]})
    with pytest.raises(WeightError, match=r"l1.mix.w2.*any"):
        load_model(tiny_vabelorn.write("worse", tmp_path, config=tiny_vabelorn.CONFIGS["A"], tensors=bad), "float32", device="cpu")


@pytest.mark.parametrize("dims,base,scaling", [(32, 20000.0, (8.0, 128, 16.0, 1.0)), (16, 100.0, (2.0, 4096, 64.0, 2.0)), (6, 50.0, (3.0, 40, 4.0, 0.5)),
                                               (2, 7.0, (1.0, 16, 2.0, 1.0)), (8, 10000.0, (16.0, 8, 2.0, 1.0)), (64, 10000.0, (6.0, 300, 3.0, 3.0))])
def test_frequencies_and_magnitude_against_the_definition(dims, base, scaling):
    want, magnitude = plain_vabelorn.yarn_frequencies(dims, base, dict(zip(("factor", "original", "fast", "slow"), scaling)))
    for cls in (PairRotarySpec, HalfRotarySpec):
        enc = POSITION_ENCODINGS.build(cls(dims=dims, base=base, yarn=tuple(float(s) for s in scaling)), torch.float32, torch.device("cpu"))
        torch.testing.assert_close(enc.inv_freq.double(), torch.tensor(want, dtype=torch.float64), atol=0.0, rtol=1e-7)
        assert enc.magnitude == pytest.approx(magnitude, abs=1e-12) == pytest.approx(0.1 * math.log(scaling[0]) + 1.0)
    plain = POSITION_ENCODINGS.build(PairRotarySpec(dims=dims, base=base), torch.float32, torch.device("cpu"))
    assert plain.magnitude == 1.0 and float(plain.inv_freq[0]) == 1.0


def test_plain_attention_depends_on_distances_only_and_adds_one():
    """What turning values and turning the sum back means: with equal queries, keys and values a shift of all positions changes nothing; and the
    weights sum to less than one."""
    g = torch.Generator().manual_seed(1)
    T, d, dv = 9, 6, 4
    q, k, v = (torch.randn(T, 1, n, generator=g, dtype=torch.float64) for n in (d, d, dv))
    fk, fv = plain_vabelorn.plain_frequencies(d, 30.0), plain_vabelorn.plain_frequencies(dv, 30.0)

    def out(shift):
        pos = torch.arange(T) + shift
        qr, kr, vr = plain_vabelorn.rotate_pairs(q, pos, fk), plain_vabelorn.rotate_pairs(k, pos, fk), plain_vabelorn.rotate_pairs(v, pos, fv)
        o = plain_vabelorn.off_by_one_attention(qr[:, 0], kr[:, 0], vr[:, 0], 0.5)
        return plain_vabelorn.rotate_pairs(o[:, None], pos, fv, sign=-1.0)[:, 0]
    torch.testing.assert_close(out(0), out(311), atol=1e-10, rtol=0.0)
    ones = plain_vabelorn.off_by_one_attention(q[:, 0], k[:, 0], torch.ones(T, 1, dtype=torch.float64), 0.5)
    assert float(ones.max()) < 1.0 and float(ones.min()) > 0.0
    s0 = float(q[0, 0] @ k[0, 0]) * 0.5
    assert float(ones[0]) == pytest.approx(math.exp(s0) / (1.0 + math.exp(s0)))


def test_cache_plan_and_slots_that_start_from_zero(cpu_ops, folders):
    _, model = load_model(folders["A"], "float32", device="cpu")
    runner = make_runner(model, page_size=4, num_pages=40, max_requests=3)
    cache = runner.cache
    assert [(g.need.plane_shapes, g.need.window, len(g.runs)) for g in cache.groups] == [(((2, 10), (2, 14)), None, 1), (((4, 8), (4, 6)), None, 1)]
    states = [c.state if c is not None else None for c in runner.caches]
    assert [None if s is None else tuple(s.shape) for s in states] == [None, (4, 3 * 7 * 7 + 42), (4, 2 * 11 * 11 + 42), None]
    runner.step([StepEntry("a", [1, 2, 3], [])])
    slot = cache.slot("a")
    assert float(states[1][slot, : 3 * 49].abs().max()) > 0 and float(states[1][slot, 3 * 49:].abs().max()) > 0
    runner.release("a")
    runner.step([StepEntry("b", [4], [])])
    assert cache.slot("b") == slot
    fresh = make_runner(model, page_size=4, num_pages=40, max_requests=3)
    fresh.step([StepEntry("b", [4], [])])
    for s, f in zip(states, fresh.caches):
        if s is not None:
            assert torch.equal(s[slot], f.state[fresh.cache.slot("b")])


@pytest.mark.parametrize("name", ["A", "B", "C"])
@pytest.mark.parametrize("mode", ["whole", "tail_singles", "portions", "mixed"])
def test_step_function_equals_plain_under_every_split(cpu_ops, folders, name, mode):
    lengths = [37, 5, 50, 1, 18, 33] if name != "B" else [75, 1, 27]
    seqs, refs = tiny_vabelorn.sequences(_weights(name), lengths, tiny_vabelorn.CONFIGS[name])
    steps = scenarios.number(getattr(scenarios, mode)(seqs) if mode != "tail_singles" else scenarios.tail_singles(seqs, tail=9))
    page = tiny_vabelorn.PAGE_SIZES[name]
    _, model = load_model(folders[name], "float32", device="cpu")
    runner = make_runner(model, page_size=page, num_pages=-(-scenarios.max_tokens_needed(steps, unit=page) // page) + 1, max_requests=4)
    scenarios.check(steps, _run(runner, steps), refs, TOL, f"{name}/{mode}")
    assert runner.cache.live_requests() == [] and runner.cache.free_pages() == runner.cache.capacity()


@pytest.mark.parametrize("seed", range(4))
def test_configurations_drawn_at_random(cpu_ops, tmp_path, seed):
    import random
    rnd = random.Random(40 + seed)
    conf = tiny_vabelorn.random_config(rnd, big=False)
    page = rnd.choice([4, 8, 16])
    tensors = tiny_vabelorn.tensors_for("", config=conf, seed=seed)
    folder = tiny_vabelorn.write(f"random{seed}", tmp_path, config=conf, tensors=tensors)
    seqs, refs = tiny_vabelorn.sequences({k: v.double() for k, v in tensors.items()}, [rnd.randint(1, 60) for _ in range(4)], conf, seed=seed)
    _, model = load_model(folder, "float32", device="cpu")
    for mode in ("portions", "mixed"):
        steps = scenarios.number(getattr(scenarios, mode)(seqs))
        runner = make_runner(model, page_size=page, num_pages=-(-scenarios.max_tokens_needed(steps, unit=page) // page) + 1, max_requests=4)
        scenarios.check(steps, _run(runner, steps), refs, TOL, f"{conf}/{mode}")
        assert runner.cache.free_pages() == runner.cache.capacity()


def test_stream_after_every_layer_against_plain(cpu_ops, folders):
    from torchlet_amd.parts.base import Stream
    ids = [5, 17, 3, 60, 2, 2, 41, 9, 30, 11, 90, 4, 4, 8]
    _, want = plain_vabelorn.forward(tiny_vabelorn.CONFIGS["A"], _weights("A"), ids)
    _, model = load_model(folders["A"], "float32", device="cpu")
    runner = make_runner(model, page_size=4, num_pages=12, max_requests=1)
    seen = []
    for block in model.blocks:
        def wrapped(stream, ctx, cache, inner=block.forward, norm=block.mixer_norm):
            stream = inner(stream, ctx, cache)
            copy = Stream(stream.residual.clone(), stream.pending)
            copy.post = stream.post
            norm.settle(copy)
            seen.append(copy.residual)
            return stream
        block.forward = wrapped
    runner.step([StepEntry("a", ids, [len(ids) - 1])])
    assert len(seen) == 4
    for got, ref in zip(seen, want):
        torch.testing.assert_close(got.double(), ref, atol=5e-5, rtol=1e-5)


def test_time_mixing_behind_a_block_that_norms_its_input(cpu_ops):
    """The mixer stands in another arrangement too: handed normed activations instead of the stream, whole and in portions."""
    from torchlet_amd.config import WKVSpec
    from torchlet_amd.engine.batch import StepContext
    from torchlet_amd.parts import MIXERS
    H, heads, dim, vdim = 12, 2, 5, 3
    spec = WKVSpec(hidden=H, heads=heads, dim=dim, vdim=vdim, decay_rank=4, norm_eps=1e-5)
    part = MIXERS.build(spec, torch.float32, torch.device("cpu"))
    g = torch.Generator().manual_seed(3)
    w = {k: torch.randn(s.shape, generator=g) * (0.4 if k not in ("norm",) else 1.0) for k, s in part.weight_specs().items()}
    part.load_weights(w)
    h = torch.randn(11, H, generator=g)

    class Cache:
        state = torch.zeros(3, heads * dim * vdim + H)

    def run(lo, hi):
        ctx = StepContext(new_lens=[hi - lo], ctx_lens=[lo], slots=[1], token_ids=[0] * (hi - lo), want_rows=[], block_tables=[], tile_sizes=set(), device="cpu")
        return part.forward(h[lo:hi], ctx, Cache)
    whole = run(0, 11)
    Cache.state.zero_()
    cut = torch.cat([run(0, 3), run(3, 4), run(4, 9), run(9, 11)])
    torch.testing.assert_close(cut, whole, atol=1e-5, rtol=1e-5)
    d = {k: v.double() for k, v in w.items()}
    x = h.double()
    mixed = {s: plain_vabelorn.token_shift(x, d[f"mu.{s}"]) for s in "rkvgw"}
    r, k = ((mixed[s] @ d[s].T).view(11, heads, dim) for s in "rk")
    v = (mixed["v"] @ d["v"].T).view(11, heads, vdim)
    decay = torch.exp(-torch.exp(torch.tanh(mixed["w"] @ d["w1"].T) @ d["w2"].T + d["w0"])).view(11, heads, dim)
    o = plain_vabelorn.rms(plain_vabelorn.wkv_recurrence(r, k, v, decay, d["u"])[0], 1e-5).reshape(11, -1)
    want = (o * d["norm"] * plain_vabelorn.silu(mixed["g"] @ d["g"].T)) @ d["o"].T
    torch.testing.assert_close(whole.double(), want, atol=1e-4, rtol=1e-4)


def _greedy(cfg, w, prompt, n):
    ids = list(prompt)
    for _ in range(n):
        ids.append(int(plain_vabelorn.forward(cfg, w, ids)[0][-1].argmax()))
    return ids[len(prompt):]


def test_greedy_generation_through_scheduler_and_sampler(cpu_ops, folders):
    """Prompts in portions of at most 12 tokens beside decode tokens, five requests over three slots (slots and pages are used again),
    steps enqueued ahead of their tokens, against the plain loop."""
    w, cfg = _weights("B"), tiny_vabelorn.CONFIGS["B"]
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
    seqs, refs = tiny_vabelorn.sequences(_weights("A"), [13, 6, 40], tiny_vabelorn.CONFIGS["A"])
    steps = scenarios.number(scenarios.mixed(seqs, seed=1))
    args = trace.parse_args(["--model", str(folders["A"]), "--dtype", "float32", "--out", str(tmp_path / "out"),
                             "--max-tokens", str(scenarios.max_tokens_needed(steps)), "--page-size", "4"])
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
    src.write_text(json.dumps(tiny_vabelorn.CONFIGS["A"]))
    assert main(["init", "--config", str(src), "--seed", "3", "--out", str(tmp_path / "out")]) == 0
    cfg = load_config(tmp_path / "out")
    assert isinstance(cfg, VabelornConfig) and cfg.layers == tiny_vabelorn.CONFIGS["A"]["layers"] and cfg.token_side == dict(dim=5)
    with safe_open(str(tmp_path / "out" / "model.safetensors"), framework="pt") as f:
        stored = set(f.keys())
    assert stored == {n for n, s in DecoderModel(cfg.to_spec(), torch.float32, "cpu").weight_specs().items() if not s.optional}
    _, model = load_model(tmp_path / "out", "float32", device="cpu")
    logits = make_runner(model, page_size=4, num_pages=8, max_requests=1).step([StepEntry("a", [1, 2, 3, 4, 5], [4])])
    assert logits.shape == (1, 97) and bool(torch.isfinite(logits).all())
