"""The Senotar decoder through the engine against the plain oracle.

Every model here is written as a checkpoint folder from its own small
configuration and random weights, and loaded the way a user loads one. The CPU
runs check the engine (caches, state slots, batches, schedules); the ``gpu`` runs
check the same through the kernels, in float32 at a tight tolerance and in bf16
at a loose one.
"""
import json
import os
import subprocess
import sys

import pytest
import torch
from safetensors.torch import save_file

import decoder_rig
import senotar_oracle as oracle
from aurora_amd import ops
from aurora_amd.engine.engine import EngineConfig, LLMEngine
from aurora_amd.engine.replay import TraceReplayer
from aurora_amd.engine.sampling_params import SamplingParams
from aurora_amd.models.config import get_spec, spec_from_checkpoint
from aurora_amd.ops import sequence

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


# ----------------------------------------------------------- small checkpoints

def mix(heads, dim, vdim, rank, scale=None, kv_from=None):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": rank,
         "scale": dim ** -0.5 if scale is None else scale}
    return m if kv_from is None else {**m, "kv_from": kv_from}


def config(name):
    """Unlike models. ``plain``: even sizes. ``odd``: sizes that fit no tile,
    unequal layers, layers without a feed-forward, latents read across other
    layers. ``single``: ones everywhere a one is allowed. ``large``: more heads
    than a tile has rows, and latents on both sides of the widest tile."""
    if name == "plain":
        layers = [(mix(4, 32, 32, 64), 96), (mix(4, 32, 32, 64), 96),
                  (mix(4, 32, 32, 64, kv_from=1), 96)]
        vocab, width, taps, emb = 333, 128, 4, (11.3, 127, 31, 5)
    elif name == "odd":
        layers = [(mix(3, 12, 40, 20, 0.41), None), (mix(5, 72, 10, 50, 0.2), 36),
                  (mix(7, 20, 24, 20, 0.3, kv_from=0), 52), (mix(1, 33, 70, 7), 20),
                  (mix(2, 40, 9, 50, 0.1, kv_from=1), None), (mix(4, 8, 8, 7, kv_from=3), 44)]
        vocab, width, taps, emb = 301, 90, 3, (0.7, 61, 1000003, 998244353)
    elif name == "single":
        layers = [(mix(1, 1, 1, 1), 1), (mix(1, 1, 1, 1, kv_from=0), None)]
        vocab, width, taps, emb = 64, 32, 1, (1.0, 1, 1, 1)
    else:
        layers = [(mix(20, 128, 64, 260), 64), (mix(2, 160, 40, 530), None),
                  (mix(33, 16, 100, 260, kv_from=0), 64)]
        vocab, width, taps, emb = 128, 192, 6, (3.0, 255, 2, 3)
    return {"architecture": "Senotar", "vocab": vocab, "width": width,
            "norm": {"eps": 1e-5}, "canon": {"taps": taps},
            "embedding": {"scale": emb[0], "bigram": {
                "buckets": emb[1], "mul_prev": emb[2], "mul_cur": emb[3]}},
            "layers": [{"type": "latent_attention", "mixer": m,
                        "mlp": None if f is None else {"kind": "dense", "ff": f}}
                       for m, f in layers]}


def weights(cfg, seed=0):
    """Random tensors, sized so that every term of the design matters: scores of
    a few units, sinks among them, gates half open, both sides of the activation."""
    gen = torch.Generator().manual_seed(seed)

    def n(*shape, s=1.0):
        return torch.randn(*shape, generator=gen) * s

    def lin(o, i, s=1.0):
        return n(o, i, s=s * i ** -0.5)

    w = cfg["width"]
    emb = cfg["embedding"]
    t = {"embed": n(cfg["vocab"], w), "head": lin(cfg["vocab"], w),
         "bigram": n(emb["bigram"]["buckets"] + 1, w, s=emb["scale"]),
         "embed.norm": 1 + n(w, s=0.2), "final.norm": 1 + n(w, s=0.2)}
    for i, layer in enumerate(cfg["layers"]):
        l, m, f = f"l{i}.", layer["mixer"], layer["mlp"]
        H, d, e, r = m["heads"], m["dim"], m["vdim"], m["kv_rank"]
        t[l + "norm1"] = 1 + n(w, s=0.2)
        t[l + "canon1"] = n(w, cfg["canon"]["taps"], s=0.5)
        t[l + "rg1"], t[l + "rg1.b"] = lin(w, w), n(w)
        p = l + "mix."
        t[p + "q"] = lin(H * d, w, 2.5 / (m["scale"] * d ** 0.5))
        if "kv_from" not in m:
            t[p + "dkv"], t[p + "dkv.norm"] = lin(r, w), 1 + n(r, s=0.3)
        t[p + "uk"], t[p + "uv"] = lin(H * d, r), lin(H * e, r)
        t[p + "sink"], t[p + "g"] = n(H, s=2.0), lin(H, w, 2.0)
        t[p + "o"] = lin(w, H * e, 2.0)
        if f is not None:
            t[l + "norm2"] = 1 + n(w, s=0.2)
            t[l + "rg2"], t[l + "rg2.b"] = lin(w, w), n(w)
            t[l + "mlp.up"], t[l + "mlp.down"] = lin(f["ff"], w, 1.5), lin(w, f["ff"])
            t[l + "mlp.act"] = n(2)
    return {k: v.to(torch.bfloat16) for k, v in t.items()}


def make_rig(path, name, device, dtype="float32"):
    cfg = config(name)
    # a latent of one number is a sign after its norm, and may fall either way
    # by rounding where it is near zero
    return decoder_rig.Rig(path, cfg, weights(cfg), oracle, device, dtype,
                           0.4 if name == "single" else 0.1)


CASES = [pytest.param((n, d, t), id=f"{n}-{d}-{t}",
                      marks=[pytest.mark.gpu] if d == "cuda" else [])
         for n in ("plain", "odd", "single", "large")
         for d, t in (("cpu", "float32"), ("cuda", "float32"), ("cuda", "bfloat16"))]


@pytest.fixture(scope="module", params=CASES)
def rig(request, tmp_path_factory):
    name, device, dtype = request.param
    if device == "cuda" and not torch.cuda.is_available():
        pytest.skip("no GPU in this container")
    return make_rig(tmp_path_factory.mktemp("ckpt"), name,
                    "auto" if device == "cuda" else "cpu", dtype)


@pytest.fixture(scope="module")
def cpu_rig(tmp_path_factory):
    return make_rig(tmp_path_factory.mktemp("ckpt"), "odd", "cpu")


# --------------------------------------------------------------- whole models

def test_whole_prompt(rig):
    toks = rig.tokens(90, 0)
    rig.check(rig.run(rig.replayer(), "a", toks, [90]), rig.logits(toks))


def test_residual_after_every_layer(rig):
    """The residual stream, layer by layer: a fault shows where it happens."""
    toks = rig.tokens(37, 1)
    want, got = oracle.forward(rig.cfg, rig.t, toks)[1], rig.trail(toks)
    assert len(got) == len(want)
    for a, b in zip(got, want):
        rig.check(a, b, 3e-5 if rig.dtype == "float32" else 0.06)


def test_token_by_token(rig):
    toks = rig.tokens(90, 0)
    rig.check(rig.run(rig.replayer(), "a", toks, [1] * 90), rig.logits(toks))


@pytest.mark.parametrize("cuts", [[2] * 45, [7, 2, 16, 1, 33, 2, 29], [64, 2, 15, 9],
                                  [1, 89], [17, 16, 1, 1, 1, 15, 39], [2, 1, 2, 85]], ids=str)
def test_portions(rig, cuts):
    toks = rig.tokens(90, 0)
    rig.check(rig.run(rig.replayer(), "a", toks, cuts), rig.logits(toks))


@pytest.mark.parametrize("n", [1, 2, 3])
def test_first_tokens(rig, n):
    """A sequence's first tokens, alone, as its whole prompt or one by one."""
    toks = rig.tokens(n, 5)
    rp = rig.replayer()
    rig.check(rig.run(rp, "a", toks, [n]), rig.logits(toks))
    rig.check(rig.run(rp, "b", toks, [1] * n), rig.logits(toks))


def test_unequal_batch(rig):
    """Prompt portions and decoded tokens in one batch, requests that pause,
    start late and end early: each as if it were alone."""
    toks = {r: rig.tokens(n, i) for i, (r, n) in
            enumerate({"a": 70, "b": 33, "c": 90, "d": 5}.items())}
    rig.run_plan(rig.replayer(max_tokens=320), toks, [
        {"a": 40, "d": 5}, {"a": 1, "b": 20}, {"b": 1, "a": 1, "c": 50},
        {"c": 2}, {"b": 1, "c": 1}, {"c": 17, "a": 1, "b": 11}, {"a": 27, "c": 20}])


def test_reused_pages_and_slots(rig):
    """One slot and a pool that only just fits, so every later request gets what
    an earlier one left behind."""
    rp = rig.replayer(max_tokens=96, requests=1)
    free = rp.engine.kv.num_free()
    for i, cuts in enumerate([[90], [5, 1, 1], [2] * 20, [1] * 12, [1], [64, 26]]):
        toks = rig.tokens(sum(cuts), 10 + i)
        rig.check(rig.run(rp, f"r{i}", toks, cuts), rig.logits(toks))
        assert rp.engine.kv.num_free() == free and rp.engine.states.num_free() == 1


def test_long_decoding(rig):
    n = 200 if rig.device == "cpu" else 400
    toks = rig.tokens(n, 3)
    rig.check(rig.run(rig.replayer(), "a", toks, [20] + [1] * (n - 20)), rig.logits(toks))


def test_greedy_generation(rig):
    """Through add_request, the scheduler (prompts cut at 32 tokens, batches of
    prompts beside decoding) and the sampler."""
    eng = rig.engine(kv_cache_pages=64, max_num_seqs=3, max_batched_tokens=32,
                     max_model_len=256)
    prompts = [rig.tokens(n, 20 + n) for n in (3, 70, 25, 40)]
    out = eng.generate(prompts, SamplingParams(max_tokens=12, **decoder_rig.GREEDY))
    assert eng.states.num_free() == eng.states.num_slots
    rig.check_greedy(prompts, out, 12)


# ----------------------------------------------------- the engine's own workings

def test_only_layers_with_latents_of_their_own_have_a_cache(cpu_rig):
    eng = cpu_rig.engine(kv_cache_pages=8, max_num_seqs=1)
    assert eng.kv.layout == [(1, 64, 0)] * 3
    assert eng.states.states[0][0].dtype == torch.int32  # the last token
    assert [s[0].shape[1:] for s in eng.states.states[1:]] == [(2, 90)] * 6


def test_preemption_recomputes_state(cpu_rig):
    eng = cpu_rig.engine(kv_cache_pages=6, max_num_seqs=2, max_model_len=80)
    prompts = [cpu_rig.tokens(20, 40), cpu_rig.tokens(18, 41)]
    out = eng.generate(prompts, SamplingParams(max_tokens=30, **decoder_rig.GREEDY))
    assert eng.counters["preemptions"] > 0
    for prompt, got in zip(prompts, out):
        assert got == cpu_rig.logits(prompt + got)[len(prompt) - 1:-1].argmax(-1).tolist()
    assert eng.kv.num_free() == 6 and eng.states.num_free() == eng.states.num_slots


def test_session_continues_from_its_state(cpu_rig):
    eng = cpu_rig.engine(kv_cache_pages=32, max_num_seqs=2, max_model_len=256)
    first = cpu_rig.tokens(21, 50)
    out = decoder_rig.turn(eng, "t1", first, 5, "s")
    assert out == cpu_rig.greedy(first, 5)
    before = eng.counters["prompt_tokens"]
    second = first + out + cpu_rig.tokens(9, 51)
    assert decoder_rig.turn(eng, "t2", second, 5, "s") == cpu_rig.greedy(second, 5)
    assert eng.counters["prompt_tokens"] - before == len(second) - (len(first) + 4)
    # departs from it: everything runs again
    third = second[:15] + cpu_rig.tokens(9, 52)
    assert decoder_rig.turn(eng, "t3", third, 5, "s") == cpu_rig.greedy(third, 5)


def test_equal_prompts_share_no_pages(cpu_rig):
    eng = cpu_rig.engine(kv_cache_pages=64, max_num_seqs=4, max_model_len=256)
    prompt = cpu_rig.tokens(50, 70)
    p = SamplingParams(max_tokens=4, **decoder_rig.GREEDY)
    assert eng.generate([prompt] * 2, p) == [cpu_rig.greedy(prompt, 4)] * 2
    assert eng.counters["prefix_cache_pages"] == 0


def test_trace_run_program(cpu_rig, tmp_path):
    toks = cpu_rig.tokens(12, 90)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": toks[:9], "want": [8, 0]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": toks[9:], "want": [2]}], "end": ["a"]}]
    r = subprocess.run(
        [sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", cpu_rig.path,
         "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "64", "--device", "cpu"],
        input="".join(json.dumps(s) + "\n" for s in steps), text=True, capture_output=True,
        timeout=120)
    assert r.returncode == 0, r.stderr
    for step, rows in ((0, [8, 0]), (1, [11])):
        raw = bytearray((tmp_path / f"{step}.f32").read_bytes())
        cpu_rig.check(torch.frombuffer(raw, dtype=torch.float32).view(len(rows), -1),
                      cpu_rig.logits(toks)[rows])


# ------------------------------------------------------- config, loader, registry

@pytest.mark.parametrize("name", ["plain", "odd", "single"])
def test_config_and_weights_round_trip(tmp_path, name):
    from aurora_amd.models.loader import save_named_safetensors
    from aurora_amd.models.registry import build_model

    rig = make_rig(tmp_path, name, "cpu")
    spec = spec_from_checkpoint(rig.path)
    assert spec.arch == "senotar" and spec.n_layers == len(rig.cfg["layers"])
    assert spec.param_count() == sum(v.numel() for v in rig.t.values())
    m = build_model(spec, torch.float32, "cpu", rig.path)
    again = m.named_tensors()
    assert set(again) == set(rig.t)
    for k, v in rig.t.items():
        assert torch.equal(again[k], v.float()), k
    (tmp_path / "copy").mkdir()
    save_named_safetensors(m, str(tmp_path / "copy"))
    m2 = build_model(spec, torch.float32, "cpu", str(tmp_path / "copy"))
    assert all(torch.equal(again[k], v) for k, v in m2.named_tensors().items())


def test_bad_configs_are_refused(tmp_path):
    cfg = config("odd")
    save_file(weights(cfg), str(tmp_path / "model.safetensors"))

    def spec(change):
        c = json.loads(json.dumps(cfg))
        change(c["layers"])
        (tmp_path / "config.json").write_text(json.dumps(c))
        return get_spec(str(tmp_path))

    assert spec(lambda ls: None).n_layers == 6
    for change in (lambda ls: ls[0].update(type="other"),
                   lambda ls: ls[1]["mlp"].update(kind="moe"),
                   lambda ls: ls[2]["mixer"].update(kv_from=2),   # itself
                   lambda ls: ls[2]["mixer"].update(kv_from=4),   # a later layer
                   lambda ls: ls[4]["mixer"].update(kv_from=2),   # one that borrows
                   lambda ls: ls[4]["mixer"].update(kv_from=0)):  # another rank
        with pytest.raises(ValueError):
            spec(change)


def test_presets_run():
    eng = LLMEngine(EngineConfig(model="tiny-senotar", device="cpu", seed=7))
    p = SamplingParams(max_tokens=6, **decoder_rig.GREEDY)
    prompts = [[5, 9, 2], list(range(40, 90)), [7] * 25]
    assert eng.generate(prompts, p) == [eng.generate([x], p)[0] for x in prompts]


@pytest.mark.gpu
def test_captured_and_eager_decoding_agree():
    """Replays of captured steps, with prompts, pauses and joins between them,
    against the same steps run eagerly."""
    from aurora_amd.models.registry import build_model

    spec = get_spec("smoke-senotar")
    model = build_model(spec, torch.bfloat16, "cuda", seed=3)
    gen = torch.Generator().manual_seed(1)
    toks = {r: torch.randint(0, spec.vocab_size, (700,), generator=gen).tolist() for r in "abc"}
    plan = ([{"a": 400}, {"b": 333}] + [{"a": 1, "b": 1}] * 20 + [{"c": 50, "a": 1}]
            + [{"a": 1, "b": 1, "c": 1}] * 20 + [{"b": 1}] * 5 + [{"c": 1, "a": 1}] * 20)

    def run(graphs):
        rp = TraceReplayer(LLMEngine(EngineConfig(
            model=spec.name, page_size=64, kv_cache_pages=64, max_num_seqs=4, state_slots=4,
            max_model_len=1024, use_hip_graphs=graphs), model=model))
        at, out = dict.fromkeys(toks, 0), []
        for step in plan:
            entries = [(r, toks[r][at[r]:at[r] + n], [n - 1]) for r, n in step.items()]
            for r, n in step.items():
                at[r] += n
            out.append(rp.step(entries).cpu())
        return torch.cat(out)

    a, b = run(True), run(False)
    assert torch.isfinite(a).all()
    # the batch is padded to its bucket in a captured step, so products may be
    # tiled otherwise; nothing else differs
    assert ((a - b).norm(dim=-1) / b.norm(dim=-1)).quantile(0.9) < 0.02


# --------------------------------------------------------- each mechanism alone

DEVICES = [pytest.param("cpu"), pytest.param("cuda", marks=pytest.mark.gpu)]
D64 = torch.float64


def _seg(n, device, start=0, pages=None, single=False, P=16):
    """The segment of one sequence's next n tokens (``single``: as a decoded one)."""
    pages = torch.arange(-(-(start + n) // P)) if pages is None else pages
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=device)  # noqa: E731
    tail = () if single else (i32([0, n]), [0, n], [start + n])
    return ops.Segment(slice(0, n), i32([pages.tolist()]), i32([start + n]), i32([start]),
                       i32([0]), *tail)


def _cuts(cuts):
    at = 0
    for c in cuts:
        yield at, at + c
        at += c


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("cuts", [[40], [1] * 40, [2, 1, 17, 1, 1, 18]], ids=len)
def test_pair_embedding_alone(device, cuts):
    """Against the oracle's rows, with factors whose product needs 64 bits and a
    table of which every row differs."""
    V, W, B = 50, 24, 13
    bigram = {"buckets": B, "mul_prev": 2 ** 40 + 9, "mul_cur": 2 ** 33 + 1}
    cfg = {"embedding": {"scale": 2.5, "bigram": bigram}, "norm": {"eps": 1e-4}}
    t = {"embed": torch.randn(V, W), "bigram": torch.randn(B + 1, W) * 3,
         "embed.norm": torch.randn(W)}
    ids = torch.randint(0, V, (40,))
    want = oracle.embed_tokens(ids.tolist(), {k: v.double() for k, v in t.items()}, cfg)
    dev = {k: v.to(device) for k, v in t.items()}
    prev = torch.full((1, 1), 7, dtype=torch.int32, device=device)  # an earlier owner's
    got = [ops.embed_pairs(ids[a:b].to(device), dev["embed"], 2.5, dev["bigram"],
                           bigram["mul_prev"], bigram["mul_cur"], dev["embed.norm"], 1e-4, prev,
                           [_seg(b - a, device, a, single=a > 0 and b - a == 1)])
           for a, b in _cuts(cuts)]
    assert (torch.cat(got).cpu() - want).abs().max() < 1e-5 * want.abs().max()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("taps", [1, 2, 4, 9])
@pytest.mark.parametrize("W", [24, 21])
def test_input_convolution_alone(device, taps, W):
    """One input far above the rest: it must show in exactly the outputs whose
    taps reach it, in portions, across their borders and in single tokens."""
    T, hit = 50, 20
    h = torch.randn(T, W)
    h[hit] *= 1000
    w = torch.randn(W, taps)
    want = oracle.add_short_conv(h.double(), w.double())
    assert (want[hit:hit + taps].abs().amax(-1) > 20).all()
    assert (want[hit + taps:].abs() < 50).all() and (want[:hit].abs() < 50).all()
    for cuts in ([T], [1] * T, [hit, 30], [hit + 1, 29], [2] * 25, [hit + taps - 1, 2, T - hit - taps - 1]):
        ring = torch.full((1, taps - 1, W), float("nan"), device=device)  # never read fresh
        got = []
        for a, b in _cuts(cuts):
            seg = _seg(b - a, device, a, single=a > 0 and b - a == 1)
            out = torch.empty(b - a, W, device=device)
            ops.short_conv_add(h[a:b].to(device), w.t().contiguous().to(device), ring, seg, out)
            got.append(out)
        err = (torch.cat(got).cpu() - want).abs().max(-1).values
        assert (err < 1e-5 * want.abs().max(-1).values.clamp(min=1)).all(), cuts


@pytest.mark.parametrize("device", DEVICES)
def test_activation_and_gated_residual_alone(device):
    z = torch.cat([torch.linspace(-30, 30, 301), torch.tensor([0.0, 1e-6, -1e-6])]).view(16, 19)
    for p, q in ((0.4, -1.3), (-30.0, 20.0)):
        want = oracle.xielu(z.double(), torch.tensor(p).double(), torch.tensor(q).double())
        got = ops.xielu(z.to(device), torch.tensor([p, q], device=device)).cpu()
        assert ((got - want).abs() < 2e-6 * (1 + want.abs())).all()
    x, y, g = torch.randn(5, 36), torch.randn(5, 36), torch.randn(5, 36) * 3
    b, w = torch.randn(36), torch.randn(36)
    want = x.double() + torch.sigmoid(g.double() + b) * y
    xs = x.to(device)
    n = ops.residual_rmsnorm(xs, w.to(device), 1e-3, delta=y.to(device), offset=0.0,
                             dtype=torch.float32, gate=(g.to(device), b.to(device)))
    assert (xs.cpu() - want).abs().max() < 1e-5
    assert (n.cpu() - oracle.weighted_norm(want, w.double(), 1e-3)).abs().max() < 1e-5


def _latents_attend(c, q, gate, uk, uv, sink, scale, rank, cuts, device, dtype, monkeypatch,
                    expand=False, P=16):
    """ops.latent_write and ops.latent_attention over the portions of ``cuts``;
    latents normed with weights that undo the norm's scale are c itself."""
    T, H, d = q.shape
    e = uv.shape[1]
    monkeypatch.setattr(sequence, "expand_latents", lambda seg, *a: expand and not seg.decode)
    R, D, E = ops.latent_width(rank), ops.latent_head_width(d), ops.latent_head_width(e)
    pages = torch.randperm(-(-T // P))
    cache = torch.full((len(pages), 1, P, R), 9.0, dtype=dtype, device=device)
    ukp, uvp = torch.zeros(H, D, R), torch.zeros(H, E, R)
    ukp[:, :d, :rank], uvp[:, :e, :rank] = uk, uv
    mv = lambda t: t.to(dtype).to(device)  # noqa: E731
    p = ops.LatentParams(H, D, E, scale, 0, H * D + rank, mv(ukp),
                         mv(ukp.transpose(1, 2).contiguous()), mv(uvp), sink.to(device))
    rows = torch.zeros(T, -(-(H * D + rank + H) // 8) * 8)
    rows[:, :H * D] = torch.nn.functional.pad(q, (0, D - d)).reshape(T, -1)
    rows[:, H * D:H * D + rank] = c
    rows[:, H * D + rank:H * D + rank + H] = gate
    rows = mv(rows)
    out = torch.zeros(T, H * E, dtype=dtype, device=device)
    for a, b in _cuts(cuts):
        slots = torch.tensor([int(pages[t // P]) * P + t % P for t in range(a, b)],
                             dtype=torch.int32, device=device)
        ops.latent_write(rows[a:b], H * D, rank, torch.ones(rank, device=device), 0.0, slots, cache)
        seg = _seg(b - a, device, a, pages, single=a > 0 and b - a == 1)
        ops.latent_attention(rows[a:b], p, cache, seg, out[a:b])
    return out.float().cpu().view(T, H, E)[..., :e]


def _unit_rms(c):
    return c / c.pow(2).mean(-1, keepdim=True).sqrt()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=str)
@pytest.mark.parametrize("H,d,e,rank", [(4, 64, 40, 64), (20, 32, 64, 100), (3, 20, 12, 530)])
def test_far_keys_stand_out(device, dtype, H, d, e, rank, monkeypatch):
    """One key whose score is far above the rest and above the sink: the query's
    output is its value, whatever the distance, at pages' and tiles' borders, in a
    prompt, at a portion's start and in decoding; and where it is still to come,
    nothing of it is seen."""
    if device == "cpu" and dtype != torch.float32:
        pytest.skip("the CPU runs in float32")
    T, i = 270, 260
    gen = torch.Generator().manual_seed(rank)
    n = lambda *s: torch.randn(*s, generator=gen)  # noqa: E731
    c = _unit_rms(n(T, rank)).to(dtype).float()
    uk, uv = n(H, d, rank) * rank ** -0.5, n(H, e, rank) * rank ** -0.5
    gate, sink = n(T, H) + 2, n(H)
    for j in (0, 1, 15, 16, 63, 64, 127, 128, 255, 256, 259, 260, 261):
        q = n(T, H, d) * 0.3
        k_j = torch.einsum("hdr,r->hd", uk, c[j])
        q[i] = 80 * k_j / k_j.pow(2).sum(-1, keepdim=True)  # scores 80 on key j
        qs, uks, uvs, gs = (x.to(dtype).float() for x in (q, uk, uv, gate))
        k = torch.einsum("hdr,tr->thd", uks.double(), c.double())
        v = torch.einsum("her,tr->the", uvs.double(), c.double())
        want = oracle.sink_attention(qs.double(), k, v, sink, 1.0)
        want = want * torch.sigmoid(gs.double()).unsqueeze(-1)
        hit = (want[i] - v[j] * torch.sigmoid(gs[i].double()).unsqueeze(-1)).abs().max()
        assert (hit < 0.02 * v[j].abs().max()) == (j <= i)
        tol = 1e-4 if dtype == torch.float32 else 0.03
        for cuts in ([T], [i, 1, 9], [i - 2, 12], [i + 1, 9]):
            for expand in (False, True) if d == 64 and dtype == torch.bfloat16 else (False,):
                got = _latents_attend(c, q, gate, uk, uv, sink, 1.0, rank, cuts, device, dtype,
                                      monkeypatch, expand)
                err = (got - want).abs().amax((1, 2)) / want.abs().max()
                assert err[i] < tol, (j, cuts, expand, float(err[i]))
                if j == 0:
                    assert err.max() < tol, (cuts, expand, err.argmax())
        if device == "cpu" and j > 16:
            break


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=str)
@pytest.mark.parametrize("sink", [-60.0, 0.0, 4.0, 60.0])
def test_sink_counts_once_and_unscaled(device, dtype, sink, monkeypatch):
    """Equal scores of zero make every weight 1 / (keys + e^sink)."""
    if device == "cpu" and dtype != torch.float32:
        pytest.skip("the CPU runs in float32")
    T, H, d, e, rank = 150, 3, 64, 64, 64
    c = _unit_rms(torch.ones(T, rank))
    q, uk, uv = torch.zeros(T, H, d), torch.randn(H, d, rank), torch.ones(H, e, rank) / rank
    want = torch.arange(1, T + 1, dtype=D64)
    want = want / (want + torch.tensor(sink, dtype=D64).exp()) * 0.5
    for cuts in ([T], [1] * 5 + [90, 1, 1, 2, 51]):
        for expand in (False, True) if dtype == torch.bfloat16 else (False,):
            got = _latents_attend(c, q, torch.zeros(T, H), uk, uv, torch.full((H,), sink), 0.25,
                                  rank, cuts, device, dtype, monkeypatch, expand)
            tol = 1e-5 if dtype == torch.float32 else 1e-2
            assert ((got - want.view(T, 1, 1)).abs() <= tol * want.view(T, 1, 1) + 1e-20).all()


@pytest.mark.gpu
@pytest.mark.parametrize("rank", [64, 512])
@pytest.mark.parametrize("order", [1, -1], ids=["rising", "falling"])
def test_scores_that_rise_or_fall_by_hundreds(rank, order, monkeypatch):
    """The softmax's reference moves many times, or never again."""
    T, H, d = 300, 2, 64
    gen = torch.Generator().manual_seed(3)
    n = lambda *s: torch.randn(*s, generator=gen)  # noqa: E731
    base = n(rank)
    ramp = torch.linspace(-3, 3, T)[:, None] * order
    c = _unit_rms(n(T, rank) + ramp * base)
    uk, uv = (n(H, 64, rank) * rank ** -0.5 for _ in "kv")
    q = torch.einsum("hdr,r->hd", uk, base).expand(T, H, d).contiguous()

    def want(dtype):
        qs, cs, ks, vs = (x.to(dtype).double() for x in (q, c, uk, uv))
        k, v = torch.einsum("hdr,tr->thd", ks, cs), torch.einsum("her,tr->the", vs, cs)
        return oracle.sink_attention(qs, k, v, torch.zeros(H), scale) * 0.5

    scale = 300.0 / float(torch.einsum("thd,hdr,sr->hts", q[:1], uk, c).abs().max())

    def got(dtype, expand=False):
        return _latents_attend(c, q, torch.zeros(T, H), uk, uv, torch.zeros(H), scale, rank,
                               [200, 1, 99], "cuda", dtype, monkeypatch, expand)

    w = want(torch.float32)
    assert (got(torch.float32) - w).abs().max() < 1e-3 * w.abs().max()
    w = want(torch.bfloat16)
    for expand in (False, True):
        y = got(torch.bfloat16, expand)
        assert torch.isfinite(y).all()
        # of 300 units of score a rounding is one or two: winners may differ
        err = ((y - w).norm(dim=-1) / w.norm(dim=-1)).flatten()
        assert err.median() < 0.2, float(err.median())


# ------------------------------------------------ the tests would notice a fault

FAULTS = {
    "no sink": ("sink_attention", lambda f: lambda q, k, v, s, c: f(q, k, v, s - 1e3, c)),
    "scaled sink": ("sink_attention", lambda f: lambda q, k, v, s, c: f(q, k, v, s * c, c)),
    "late key": ("sink_attention", lambda f: lambda q, k, v, s, c: f(q, k.roll(1, 0), v, s, c)),
    "swapped pair": ("bigram_row", lambda f: lambda p, t, c: f(p, t, c) if p is None else f(t, p, c)),
    "first pair": ("bigram_row", lambda f: lambda p, t, c: 0 if p is None else f(p, t, c)),
    "turned taps": ("add_short_conv", lambda f: lambda h, w: f(h, w.flip(1))),
    "no past": ("add_short_conv", lambda f: lambda h, w: torch.cat([f(h[:64], w), f(h[64:], w)])),
    "raw latents": ("latents", lambda f: lambda u, t, p, e: u @ t[p + "dkv"].T),
    "open gates": ("gate", lambda f: lambda h, t, n: torch.ones_like(h)),
    "swapped slopes": ("xielu", lambda f: lambda z, p, q: f(z, q, p)),
}


@pytest.mark.parametrize("fault", list(FAULTS))
def test_a_planted_fault_shows(cpu_rig, monkeypatch, fault):
    """Each of these changes in the oracle moves its logits far beyond the
    tolerance, so the comparisons above cannot pass with such a fault."""
    toks = cpu_rig.tokens(90, 0)
    good = cpu_rig.logits(toks)
    name, change = FAULTS[fault]
    monkeypatch.setattr(oracle, name, change(getattr(oracle, name)))
    bad = oracle.forward(cpu_rig.cfg, cpu_rig.t, toks)[0]
    assert ((bad - good).norm(dim=-1) / good.norm(dim=-1)).max() > 5e-3


@pytest.mark.parametrize("change", [
    lambda ls: ls[2]["mixer"].pop("kv_from") and None,
    lambda ls: ls[4]["mixer"].update(scale=0.11)])
def test_a_change_of_one_layer_shows(cpu_rig, change):
    cfg = json.loads(json.dumps(cpu_rig.cfg))
    change(cfg["layers"])
    t = dict(cpu_rig.t)
    t["l2.mix.dkv"], t["l2.mix.dkv.norm"] = t["l0.mix.dkv"], t["l0.mix.dkv.norm"]
    toks = cpu_rig.tokens(90, 0)
    good, bad = cpu_rig.logits(toks), oracle.forward(cfg, t, toks)[0]
    assert ((bad - good).norm(dim=-1) / good.norm(dim=-1)).max() > 5e-3
