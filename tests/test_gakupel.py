"""The Gakupel decoder through the engine against the plain oracle.

Every model here is written as a checkpoint folder from its own small
configuration and random weights, and loaded the way a user loads one. The CPU
runs check the engine (caches, state slots, batches, schedules); the ``gpu`` runs
check the same through the kernels, in float32 at a tight tolerance and in bf16
at a loose one.
"""
import json
import math
import os
import subprocess
import sys

import pytest
import torch
from safetensors.torch import save_file

import decoder_rig
import gakupel_oracle as oracle
from aurora_amd import ops
from aurora_amd.engine.engine import EngineConfig, LLMEngine
from aurora_amd.engine.replay import TraceReplayer
from aurora_amd.engine.sampling_params import SamplingParams
from aurora_amd.models.config import get_spec, spec_from_checkpoint
from aurora_amd.ops import sequence, torch_ref

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


# ----------------------------------------------------------- small checkpoints

def attention(heads, kv, dim, rot, base=1e4, scale=None):
    return "attention", {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim,
                         "scale": dim ** -0.5 if scale is None else scale,
                         "rot": {"base": base, "dims": rot}}


def delta(heads, kv, dim, vdim, conv=4):
    return "delta", {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv}


def parallel(left, right, scale, temp, cap, scales):
    h, g, d, e = left
    H, D, E = right
    return "parallel", {
        "left": {"heads": h, "kv_heads": g, "dim": d, "vdim": e, "scale": scale,
                 "q_temp": {"coef": temp[0], "every": temp[1]}},
        "right": {"heads": H, "dim": D, "vdim": E, "gate_cap": cap},
        "left_scale": scales[0], "right_scale": scales[1]}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, groups, keep, ff, shared, scale=1.7):
    return {"kind": "moe", "expert": {"ff": ff}, "shared": {"ff": shared},
            "router": {"experts": experts, "top": top, "scale": scale,
                       "groups": {"count": groups, "keep": keep}}}


def config(name):
    """Unlike models. ``plain``: even sizes, every kind of layer. ``odd``: sizes that
    fit no tile, unequal layers, layers without a feed-forward, groups of one expert.
    ``single``: ones everywhere a one is allowed. ``large``: heads and states wider
    than the matrix-core attention kernels or a wave take."""
    if name == "plain":
        layers = [(delta(4, 2, 32, 64), moe(8, 2, 4, 2, 64, 128)),
                  (parallel((4, 4, 64, 64), (2, 64, 32), 0.15, (0.4, 16), 9.0, (1.3, 0.6)),
                   dense(192)),
                  (attention(6, 3, 64, 32), dense(128))]
        vocab, width, eps = 333, 128, 1e-5
    elif name == "odd":
        layers = [(attention(3, 1, 20, 6, 500.0, 0.3), moe(6, 3, 6, 4, 20, 28)),
                  (parallel((5, 1, 33, 41), (3, 10, 21), 0.21, (1.5, 7), 3.0, (0.5, 2.0)), None),
                  (delta(6, 2, 12, 7, 3), dense(37)),
                  (parallel((2, 2, 72, 9), (1, 24, 50), 0.1, (-0.2, 1), 15.0, (1.0, 1.0)),
                   moe(9, 4, 3, 2, 36, 10)),
                  (delta(3, 1, 40, 18, 2), None),
                  (attention(4, 2, 48, 48, 1e6), moe(5, 2, 1, 1, 12, 52, 0.8))]
        vocab, width, eps = 301, 90, 1e-3
    elif name == "single":
        layers = [(attention(1, 1, 2, 2), moe(1, 1, 1, 1, 1, 1)),
                  (delta(1, 1, 1, 1, 1), dense(1)),
                  (parallel((1, 1, 1, 1), (1, 1, 1), 1.0, (1.0, 1), 1.0, (1.0, 1.0)), None)]
        vocab, width, eps = 64, 32, 1.0  # else a head of one number is a sign
    else:
        layers = [(parallel((3, 1, 160, 300), (2, 70, 260), 0.08, (0.3, 33), 12.0, (0.9, 1.1)),
                   moe(70, 6, 10, 3, 64, 64)),
                  (delta(2, 1, 200, 130), None),
                  (attention(8, 1, 136, 136), dense(64))]
        vocab, width, eps = 128, 192, 1e-5
    return {"architecture": "Gakupel", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "layers": [{"type": m[0], "mixer": m[1], "mlp": f} for m, f in layers]}


def weights(cfg, seed=0, decided=False):
    """Random tensors, sized so that every term of the design matters: scores and
    distance penalties of a few units, decays of every reach, gates half open,
    corrections that change the choice (``decided``: that alone make it, so far are they
    apart), depth averages of everything so far."""
    gen = torch.Generator().manual_seed(seed)

    def n(*shape, s=1.0):
        return torch.randn(*shape, generator=gen) * s

    def lin(o, i, s=1.0):
        return n(o, i, s=s * i ** -0.5)

    w = cfg["width"]
    t = {"embed": n(cfg["vocab"], w), "head": lin(cfg["vocab"], w),
         "final.norm": 1 + n(w, s=0.2), "final.norm.b": n(w, s=0.3)}

    def heads(p, m):
        d, H, G = m["dim"], m["heads"], m["kv_heads"]
        t[p + "q"], t[p + "k"] = lin(H * d, w), lin(G * d, w)
        t[p + "o"] = lin(w, H * m["vdim"], 2.0)
        return d, H, G

    def glu(p, ff):
        t[p + "gate"], t[p + "up"], t[p + "down"] = lin(ff, w, 2.0), lin(ff, w), lin(w, ff)

    for i, layer in enumerate(cfg["layers"]):
        l, m, f = f"l{i}.", layer["mixer"], layer["mlp"]
        t[l + "norm1"], t[l + "norm1.b"] = 1 + n(w, s=0.2), n(w, s=0.2)
        t[l + "dwa"] = n(i + 2, s=0.4)
        t[l + "dwa"][-1] += 0.8
        p = l + "mix."
        if layer["type"] == "attention":
            d, _, _ = heads(p, m)
            t[p + "q.norm"] = (2 + n(d, s=0.3)) / (m["scale"] * d ** 0.5) ** 0.5
            t[p + "k.norm"] = (1 + n(d, s=0.3)) / (m["scale"] * d ** 0.5) ** 0.5
        elif layer["type"] == "delta":
            d, H, G, e, taps = m["dim"], m["heads"], m["kv_heads"], m["vdim"], m["conv"]
            for x, c in (("q", G * d), ("k", G * d), ("v", H * e)):
                t[p + x], t[p + x + ".conv"] = lin(c, w, 1.5), n(c, taps, s=0.6)
            t[p + "b"], t[p + "a"], t[p + "g"] = lin(H, w), lin(H, w), lin(H * e, w)
            t[p + "A_log"], t[p + "dt_bias"] = n(H, s=0.7) - 1, n(H) - 2
            t[p + "norm"], t[p + "o"] = 1 + n(e, s=0.2), lin(w, H * e, 2.0)
        else:
            left, right = m["left"], m["right"]
            d, H, G = heads(p + "left.", left)
            t[p + "left.v"] = lin(G * left["vdim"], w)
            s = (left["scale"] * d ** 0.5) ** -0.5
            t[p + "left.q.norm"] = (2 + n(H * d, s=0.3)) * s
            t[p + "left.k.norm"] = (1 + n(G * d, s=0.3)) * s
            t[p + "left.r1"], t[p + "left.r2"] = n(H).abs() + 0.1, n(H, s=0.3).abs() + 0.02
            p += "right."
            H, d, e = right["heads"], right["dim"], right["vdim"]
            for x, c in (("q", H * d), ("k", H * d), ("v", H * e), ("g", H * e), ("i", H), ("f", H)):
                t[p + x] = lin(c, w, 1.5)
            t[p + "i.b"], t[p + "f.b"] = n(H), n(H) + 3
            t[p + "norm"], t[p + "o"] = 1 + n(H * e, s=0.2), lin(w, H * e, 2.0)
        if f is None:
            continue
        t[l + "norm2"], t[l + "norm2.b"] = 1 + n(w, s=0.2), n(w, s=0.2)
        p = l + "mlp."
        if f["kind"] == "dense":
            t[p + "up"], t[p + "down"] = lin(f["ff"], w, 1.5), lin(w, f["ff"])
            continue
        E = f["router"]["experts"]
        t[p + "router"], t[p + "correction"] = lin(E, w, 1.5), n(E, s=0.2) - 0.8
        if decided:
            # groups one above the other, so that their sums are far apart as well
            c = f["router"]["groups"]["count"]
            rank = torch.argsort(torch.rand(c, E // c, generator=gen)) * 2.0
            t[p + "correction"] = (rank + torch.randperm(c, generator=gen).view(c, 1)
                                   * (4.0 * (E // c))).flatten() - 2 * E
        for e in range(E):
            glu(f"{p}e{e}.", f["expert"]["ff"])
        glu(p + "shared.", f["shared"]["ff"])
        t[p + "shared.sg"] = lin(1, w, 2.0)
    return {k: v.to(torch.bfloat16) for k, v in t.items()}


def make_rig(path, name, device, dtype="float32"):
    cfg = config(name)
    # in 16 bits choices that are close may fall otherwise: there, corrections decide
    t = weights(cfg, decided=dtype != "float32")
    # narrow heads whose sum nearly cancels before their norm lose most bits
    tol = {"odd": 0.3, "single": 0.3}.get(name, 0.06)
    return decoder_rig.Rig(path, cfg, t, oracle, device, dtype, tol)


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
        rig.check(a, b, 3e-5 if rig.dtype == "float32" else None)


def test_token_by_token(rig):
    toks = rig.tokens(90, 0)
    rig.check(rig.run(rig.replayer(), "a", toks, [1] * 90), rig.logits(toks))


@pytest.mark.parametrize("cuts", [[2] * 45, [7, 2, 16, 1, 33, 2, 29], [64, 2, 15, 9],
                                  [1, 89], [17, 16, 1, 1, 1, 15, 39]], ids=str)
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

def test_caches_and_states_of_the_layers(cpu_rig):
    eng = cpu_rig.engine(kv_cache_pages=8, max_num_seqs=1)
    assert eng.kv.layout == [(1, 20, 20), (1, 33, 41), (2, 72, 9), (2, 48, 48)]
    assert [[tuple(t.shape[1:]) for t in run] for run in eng.states.states] == [
        [(3, 10, 21), (3, 10), (3,)], [(6, 12, 7), (3, 90)], [(1, 24, 50), (1, 24), (1,)],
        [(3, 40, 18), (2, 134)]]


def test_preemption_recomputes_state(cpu_rig):
    eng = cpu_rig.engine(kv_cache_pages=6, max_num_seqs=2, max_model_len=80)
    prompts = [cpu_rig.tokens(20, 40), cpu_rig.tokens(18, 41)]
    out = eng.generate(prompts, SamplingParams(max_tokens=30, **decoder_rig.GREEDY))
    assert eng.counters["preemptions"] > 0
    cpu_rig.check_greedy(prompts, out, 30)
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
    third = second[:15] + cpu_rig.tokens(9, 52)  # departs from it: all runs again
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

@pytest.mark.parametrize("name", ["plain", "odd", "single", "large"])
def test_config_and_weights_round_trip(tmp_path, name):
    from aurora_amd.models.loader import save_named_safetensors
    from aurora_amd.models.registry import build_model

    rig = make_rig(tmp_path, name, "cpu")
    spec = spec_from_checkpoint(rig.path)
    assert spec.arch == "gakupel" and spec.n_layers == len(rig.cfg["layers"])
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
                   lambda ls: ls[2]["mlp"].update(kind="other"),
                   lambda ls: ls[0]["mixer"].update(vdim=10),            # values are keys
                   lambda ls: ls[0]["mixer"]["rot"].update(dims=22),     # wider than a head
                   lambda ls: ls[0]["mixer"].update(kv_heads=2),         # 3 query heads
                   lambda ls: ls[2]["mixer"].update(kv_heads=4),
                   lambda ls: ls[3]["mlp"]["router"].update(top=7),      # 6 stay open
                   lambda ls: ls[3]["mlp"]["router"]["groups"].update(count=2)):
        with pytest.raises(ValueError):
            spec(change)


def test_presets_run():
    eng = LLMEngine(EngineConfig(model="tiny-gakupel", device="cpu", seed=7))
    p = SamplingParams(max_tokens=6, **decoder_rig.GREEDY)
    prompts = [[5, 9, 2], list(range(40, 90)), [7] * 25]
    assert eng.generate(prompts, p) == [eng.generate([x], p)[0] for x in prompts]


@pytest.mark.gpu
def test_captured_and_eager_decoding_agree():
    """Replays of captured steps, with prompts, pauses and joins between them,
    against the same steps run eagerly."""
    from aurora_amd.models.registry import build_model

    spec = get_spec("smoke-gakupel")
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
    assert ((a - b).norm(dim=-1) / b.norm(dim=-1)).quantile(0.9) < 0.03


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


def _columns(**parts):
    """Named [T, n] tensors side by side, each from a multiple of 8 on."""
    at, rows, n = {}, [], 0
    for name, x in parts.items():
        at[name] = n
        rows.append(torch.nn.functional.pad(x, (0, -x.shape[1] % 8)))
        n += rows[-1].shape[1]
    return at, torch.cat(rows, 1)


def _params_to(p, dev):
    return type(p)(**{k: v.to(dev) if torch.is_tensor(v) else v for k, v in vars(p).items()})


def _attend(q, k, v, cuts, device, dtype, *, scale, whole=False, wq=None, wk=None, rot=None,
            temp=None, r1=None, r2=None, sink=False, eps=1e-6, P=16):
    """Queries, keys and values [T, heads, d] as projected, through ops.normed_qkv and
    ops.biased_attention in portions; values None: the keys."""
    T, H, d = q.shape
    G, e = k.shape[1], d if v is None else v.shape[2]
    parts = {"q": q.flatten(1), "k": k.flatten(1)}
    if v is not None:
        parts["v"] = v.flatten(1)
    at, rows = _columns(**parts)
    rows = rows.to(dtype).to(device)
    f32 = lambda t: t.float().to(device)  # noqa: E731
    ones = lambda h: torch.ones(h * d if whole else d)  # noqa: E731
    p = ops.NormedHeadsParams(
        H, G, d, e, at["q"], at["k"], at.get("v", at["k"]),
        f32(ones(H) if wq is None else wq), f32(ones(G) if wk is None else wk), whole, eps,
        None if rot is None else torch_ref.rope_cos_sin_cache(rot[0], T, rot[1]).to(device),
        temp)
    pages = torch.randperm(-(-T // P))
    DK, DV = ops.cache_head_dims(d, e, dtype, device)
    kc, vc = (torch.full((len(pages), G, P, w), 9.0, dtype=dtype, device=device)
              for w in (DK, DV))
    out = torch.zeros(T, H * e, dtype=dtype, device=device)
    slopes = f32(torch.zeros(H) if r1 is None else r1)
    for a, b in _cuts(cuts):
        pos = torch.arange(a, b, dtype=torch.int32, device=device)
        slots = torch.tensor([int(pages[t // P]) * P + t % P for t in range(a, b)],
                             dtype=torch.int32, device=device)
        qs = ops.normed_qkv(rows[a:b], p, pos, slots, kc, vc)
        ops.biased_attention(qs, kc, vc, _seg(b - a, device, a, pages, a > 0 and b - a == 1),
                             scale, 0, slopes, out[a:b], 0, e, 1.0,
                             None if r2 is None else f32(r2),
                             torch.zeros(H, device=device) if sink else None)
    return out.float().cpu().view(T, H, e)


HEADS = [(4, 2, 64, None), (3, 1, 20, 30), (8, 2, 128, 64), (2, 2, 160, 24)]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=str)
@pytest.mark.parametrize("H,G,d,e", HEADS)
def test_far_keys_stand_out(device, dtype, H, G, d, e):
    """One key in the query's own direction, far above the rest, the penalty and the
    sink: the query's output is its value, whatever the distance, at pages' and tiles'
    borders, in a prompt, at a portion's start and in decoding; and where it is still
    to come, nothing of it is seen."""
    if device == "cpu" and dtype != torch.float32:
        pytest.skip("the CPU runs in float32")
    T, i, whole = 270, 260, e is not None
    gen = torch.Generator().manual_seed(d)
    n = lambda *s: torch.randn(*s, generator=gen).to(dtype).float()  # noqa: E731
    k = n(T, G, d)
    v = None if e is None else n(T, G, e)
    r1, r2 = torch.rand(H, generator=gen) + 0.5, torch.rand(H, generator=gen)
    for j in (0, 1, 15, 16, 63, 64, 127, 128, 255, 256, 259, 260, 261):
        q = n(T, H, d)
        q[i] = k[j].repeat_interleave(H // G, 0)
        norm = oracle.whole_norm if whole else oracle.head_norm
        one = torch.ones((), dtype=D64)
        scale = 150.0 / d
        bias = (lambda h, x: oracle.log_distance(r1[h].double(), r2[h].double(), x)) \
            if whole else None
        want = oracle.attend(norm(q.double(), one if not whole else one.expand(H * d), 1e-6),
                             norm(k.double(), one if not whole else one.expand(G * d), 1e-6),
                             (k if v is None else v).double(), scale, bias, whole)
        vj = (k if v is None else v)[j].double().repeat_interleave(H // G, 0)
        hit = (want[i] - vj).abs().max() / vj.abs().max()
        assert (hit < 0.02) == (j <= i), (j, float(hit))
        tol = 1e-4 if dtype == torch.float32 else 0.04
        extra = dict(r1=r1, r2=r2, sink=True) if whole else {}
        for cuts in ([T], [i, 1, 9], [i - 2, 12], [i + 1, 9]):
            got = _attend(q, k, v, cuts, device, dtype, scale=scale, whole=whole, **extra)
            err = (got - want).abs().amax((1, 2)) / want.abs().max()
            assert err[i] < tol, (j, cuts, float(err[i]))
        if device == "cpu" and j > 16:
            break


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=str)
@pytest.mark.parametrize("d", [64, 40, 200])
def test_distance_and_sink_have_closed_forms(device, dtype, d):
    """Scores of zero and values of one leave Z / (1 + Z), Z the sum of
    (1 + b distance)^-a over the keys."""
    if device == "cpu" and dtype != torch.float32:
        pytest.skip("the CPU runs in float32")
    T, H, e = 300, 5, 64
    r1 = torch.tensor([0.0, 1.0, 0.5, 6.0, -0.5])
    r2 = torch.tensor([0.3, 0.0, 0.7, 0.01, 0.02])
    q, k, v = torch.zeros(T, H, d), torch.randn(T, H, d), torch.ones(T, H, e)
    dist = torch.arange(T, dtype=D64)
    want = ((1 + r2.double() * dist[:, None]) ** -r1.double()).cumsum(0)
    tol = 2e-5 if dtype == torch.float32 else 1e-2
    for cuts in ([T], [1] * 5 + [90, 1, 1, 2, 201]):
        for sink in (True, False):
            got = _attend(q, k, v, cuts, device, dtype, scale=0.3, whole=True, r1=r1, r2=r2,
                          sink=sink)
            w = want / (want + 1) if sink else torch.ones_like(want)
            assert ((got - w.unsqueeze(-1)).abs() < tol).all(), (cuts, sink)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,d,rot", [(4, 2, 64, 64), (4, 2, 64, 16), (3, 1, 20, 6), (2, 1, 2, 2)])
def test_rotation_and_head_norm_alone(device, H, G, d, rot):
    """Far positions, whose angles need all of their bits; norms of tiny heads, where
    the epsilon matters; values that are the keys before both."""
    T, base, eps = 40, 300.0, 1e-3
    q, k = torch.randn(T, H, d), torch.randn(T, G, d)
    k[::3] *= 0.01
    wq, wk = torch.randn(d), torch.randn(d)
    start = 900
    pad = lambda x: torch.cat([torch.zeros(start, *x.shape[1:], dtype=D64), x])  # noqa: E731
    turn = lambda x: oracle.rotate(pad(x), rot, base)[start:]  # noqa: E731
    wants = [turn(oracle.head_norm(x.double(), w.double(), eps)) for x, w in ((q, wq), (k, wk))]
    at, rows = _columns(q=q.flatten(1), k=k.flatten(1))
    p = _params_to(ops.NormedHeadsParams(
        H, G, d, d, at["q"], at["k"], at["k"], wq, wk, False, eps,
        torch_ref.rope_cos_sin_cache(rot, 1024, base), None), device)
    kc, vc = (torch.zeros(T, G, 1, d, device=device) for _ in "kv")
    pos = torch.arange(start, start + T, dtype=torch.int32, device=device)
    got = ops.normed_qkv(rows.to(device), p, pos, pos - start, kc, vc)
    for a, b in ((got, wants[0]), (kc[:, :, 0], wants[1]), (vc[:, :, 0], k)):
        assert (a.cpu() - b).abs().max() < 1e-5 * max(1.0, float(b.abs().max()))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("every", [1, 7, 64])
def test_query_temperature_steps_where_it_should(device, every):
    T, H, d = 200, 2, 24
    q, wq = torch.randn(T, H, d), torch.randn(H * d)
    at, rows = _columns(q=q.flatten(1), k=torch.randn(T, d), v=torch.randn(T, d))
    p = _params_to(ops.NormedHeadsParams(
        H, 1, d, d, at["q"], at["k"], at["v"], wq, torch.ones(d), True, 1e-6, None,
        (0.7, every)), device)
    kc, vc = (torch.zeros(T, 1, 1, d, device=device) for _ in "kv")
    pos = torch.arange(T, dtype=torch.int32, device=device)
    got = ops.normed_qkv(rows.to(device), p, pos, pos, kc, vc).cpu()
    factor = torch.tensor([oracle.temperature(t, {"coef": 0.7, "every": every})
                           for t in range(T)], dtype=D64)
    want = oracle.whole_norm(q.double(), wq.double(), 1e-6) * factor.view(T, 1, 1)
    assert (got - want).abs().max() < 2e-5
    # one position off would show
    assert (factor[every - 1] - factor[max(every - 2, 0)]).abs() > 0.4 or every == 1


def _recur(run, parts, cuts, device, state, width, op):
    """A recurrence in portions over one slot that an earlier owner left full."""
    at, rows = _columns(**parts)
    p = _params_to(run(at), device)
    states = [torch.full(s, float("nan"), device=device) for s in state]
    out = torch.zeros(rows.shape[0], width, device=device)
    for a, b in _cuts(cuts):
        op(rows[a:b].to(device), p, *states, _seg(b - a, device, a, single=a > 0 and b - a == 1),
           out[a:b], 0, 1.0)
    return out.cpu()


CUTS = [[150], [1] * 150, [2] * 75, [16, 1, 15, 64, 54], [33, 2, 1, 1, 17, 96]]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,d,e,taps", [(4, 2, 32, 24, 4), (3, 1, 20, 7, 3), (1, 1, 1, 1, 1)])
@pytest.mark.parametrize("reach", [-7.0, 0.0, 4.0])
def test_delta_rule_alone(device, H, G, d, e, taps, reach):
    """Decays of nearly one, moderate, and of nearly nothing; one token whose key comes
    back at the end, and one input so small that the unit norm's epsilon matters."""
    T, eps = 150, 1e-6
    gen = torch.Generator().manual_seed(d)
    n = lambda *s: torch.randn(*s, generator=gen)  # noqa: E731
    q, k, v, g = n(T, G * d), n(T, G * d), n(T, H * e), n(T, H * e)
    v[17] *= 30
    q[140 - taps:142] = k[17]
    k[60:66] *= 1e-4
    a, b = n(T, H), n(T, H) * 2
    conv = [n(c, taps) * 0.7 for c in (G * d, G * d, H * e)]
    a_log, dt, norm = n(H) * 0.3, n(H) + reach, 1 + n(e) * 0.2
    D = lambda *xs: [x.double() for x in xs]  # noqa: E731
    qd, kd, vd = (oracle.short_conv(x, w) for x, w in zip(D(q, k, v), D(*conv)))
    rep = lambda x: oracle.unit(x.reshape(T, G, d)).repeat_interleave(H // G, 1)  # noqa: E731
    decay = oracle.head_decay(a.double(), {"A_log": a_log.double(), "dt_bias": dt.double(),
                                           "a": torch.eye(H, dtype=D64)}, "")
    want = oracle.delta_rule(rep(qd) * d ** -0.5, rep(kd), vd.reshape(T, H, e), decay,
                             torch.sigmoid(b.double()))
    want = oracle.rms(want, eps) * norm.double() * oracle.silu(g.double()).reshape(T, H, e)
    for cuts in CUTS:
        got = _recur(lambda at: ops.HeadDeltaParams(
            H, G, d, e, taps, *(at[x] for x in "qkvbag"), torch.cat(conv), a_log, dt, norm, eps),
            dict(q=q, k=k, v=v, b=b, a=a, g=g), cuts, device,
            [(1, H, d, e), (1, taps, 2 * G * d + H * e)], H * e, ops.head_delta_rule)
        err = (got - want.flatten(1)).abs()
        # a head of one number is a sign after its norm
        assert (err.max() if e > 1 else err.quantile(0.95)) < 2e-4 * want.abs().max(), cuts


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,d,e", [(4, 32, 24), (3, 20, 15), (2, 64, 16), (1, 1, 1)])
@pytest.mark.parametrize("kind", ["mixed", "keeps", "forgets", "rises", "falls", "quiet"])
def test_matrix_memory_alone(device, H, d, e, kind):
    """Gates of every kind: memories that keep or forget all, input gates that rise or
    fall through their whole range (the running maximum moves always, or stays), and
    ones so small that the denominator is the bound's; one token that stands out."""
    T, eps, cap = 150, 1e-6, 8.0
    gen = torch.Generator().manual_seed(d)
    n = lambda *s: torch.randn(*s, generator=gen)  # noqa: E731
    q, k, v, g = n(T, H * d), n(T, H * d), n(T, H * e), n(T, H * e)
    i, f = n(T, H) * 3, n(T, H) * 2 + 3
    ramp = torch.linspace(-30, 30, T).unsqueeze(1)
    if kind == "keeps":
        f = f + 30
        i[40] = 40.0  # the cap of all others' gates
        q[149] = k[40] * 5
    elif kind == "forgets":
        f = f - 20
    elif kind == "rises":
        i = i + ramp
    elif kind == "falls":
        i = i - ramp
    elif kind == "quiet":
        i = i - 20
    ib, fb, norm = n(H), n(H), 1 + n(H * e) * 0.2
    D = lambda x, w: x.double().reshape(T, H, w)  # noqa: E731
    gates = [oracle.soft_cap(x.double() + b.double(), cap) for x, b in ((i, ib), (f, fb))]
    o = oracle.matrix_memory(D(q, d) * d ** -0.5, D(k, d), D(v, e), gates[0],
                             -oracle.softplus(-gates[1]))
    want = oracle.rms(o, eps).flatten(1) * norm.double() * torch.sigmoid(g.double())
    if kind == "keeps" and d > 1:
        v40 = oracle.rms(D(v, e)[40], eps).flatten() * norm.double() * torch.sigmoid(g[149].double())
        assert (want[149] - v40).abs().max() < 0.4 * v40.abs().max()
    for cuts in CUTS:
        got = _recur(lambda at: ops.MatrixMemoryParams(
            H, d, e, *(at[x] for x in "qkvifg"), ib, fb, norm, cap, eps),
            dict(q=q, k=k, v=v, i=i, f=f, g=g), cuts, device,
            [(1, H, d, e), (1, H, d), (1, H)], H * e, ops.matrix_memory)
        err = (got - want).abs()
        assert (err.max() if e > 1 else err.quantile(0.95)) < 5e-4 * want.abs().max(), \
            (cuts, float(err.max()))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("E,groups,keep,top", [(8, 4, 2, 3), (12, 2, 1, 6), (6, 6, 2, 2),
                                               (9, 3, 3, 4), (5, 1, 1, 5), (1, 1, 1, 1)])
def test_grouped_routing_alone(device, E, groups, keep, top):
    """Against the oracle's dense weights, with corrections that make all choice scores
    negative, and the best expert of all alone in a group that loses."""
    T, W = 64, 48
    h, router = torch.randn(T, W), torch.randn(E, W) * 0.4
    corr = torch.randn(E) * 0.3 - 1.5
    if groups > 1 and E > groups:
        corr[0] += 0.4
        corr[1:E // groups] -= 3.0
    cfg = {"top": top, "scale": 2.2, "groups": {"count": groups, "keep": keep}}
    want = oracle.route(h.double() @ router.double().T, corr.double(), cfg)
    m = torch_ref if device == "cpu" else sequence._hip("test")
    sel, w = m.moe_route_grouped(*(x.to(device) for x in (h, router, corr)), top, groups, keep, 2.2)
    got = torch.zeros(T, E, dtype=D64).scatter_(1, sel.cpu().long(), w.cpu().double())
    assert (got - want).abs().max() < 1e-5
    if groups > keep and E > groups:
        s = torch.sigmoid(h.double() @ router.double().T) + corr
        assert (want[torch.arange(T), s.argmax(-1)] == 0).any()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("W", [64, 50])
def test_output_norm_and_depth_average_alone(device, W):
    """Layer after layer: each result kept, the sum of all of them going on, a result
    of large mean and small spread in between, the final norm in the last."""
    T, n, eps = 6, 5, 1e-3
    r = [torch.randn(T, W) for _ in range(n)]
    r[2] = r[2] * 0.01 + 5.0
    ws, bs = torch.randn(n, W), torch.randn(n, W)
    cs = [torch.randn(i + 2) for i in range(n)]
    final = (torch.randn(W), torch.randn(W))
    x = torch.randn(T, W)
    kept = [x.double()]
    y = kept[0]
    buf = torch.zeros(n, T, W, device=device)
    src, out = buf[0].copy_(x), torch.empty(T, W, device=device)
    for i in range(n):
        kept.append(y + oracle.layer_norm(r[i].double(), ws[i].double(), bs[i].double(), eps))
        y = oracle.depth_average(kept, cs[i].double())
        h = ops.output_norm(src, out, ws[i].to(device), bs[i].to(device), eps,
                            delta=r[i].to(device), depth=(buf, cs[i].to(device)),
                            final=tuple(t.to(device) for t in final) if i == n - 1 else None,
                            dtype=torch.float32)
        src = out
        assert (out.cpu() - y).abs().max() < 2e-5 * y.abs().max()
    want = oracle.layer_norm(y, final[0].double(), final[1].double(), eps)
    assert (h.cpu() - want).abs().max() < 5e-5 * want.abs().max()


@pytest.mark.parametrize("device", DEVICES)
def test_activations_alone(device):
    z = torch.cat([torch.linspace(-30, 30, 301), torch.tensor([0.0, 1e-6, -1e-6])]).view(16, 19)
    assert (ops.gelu(z.to(device)).cpu() - oracle.gelu(z.double())).abs().max() < 4e-6
    u = torch.randn(16, 19)
    got = ops.silu_glu(torch.cat([z, u], 1).to(device), 19).cpu()
    assert (got - oracle.silu(z.double()) * u).abs().max() < 1e-5


# ------------------------------------------------ the tests would notice a fault

FAULTS = {
    "sink left out": ("attend", lambda f: lambda q, k, v, c, b=None, s=False: f(q, k, v, c, b)),
    "sink everywhere": ("attend", lambda f: lambda q, k, v, c, b=None, s=False: f(q, k, v, c, b, True)),
    "late key": ("attend", lambda f: lambda q, k, v, c, b=None, s=False: f(q, k.roll(1, 0), v, c, b, s)),
    "distance one off": ("log_distance", lambda f: lambda a, b, x: f(a, b, x + 1)),
    "linear distance": ("log_distance", lambda f: lambda a, b, x: a * b * x),
    "temperature one late": ("temperature", lambda f: lambda p, c: f(p - 1, c)),
    "norm per head": ("whole_norm", lambda f: lambda x, w, e: oracle.rms(x, e) * w.view(x.shape[1:])),
    "no head norm": ("head_norm", lambda f: lambda x, w, e: x * w),
    "other rotation": ("rotate", lambda f: lambda x, n, b: f(x, n, b * 1.5)),
    "interleaved pairs": ("rotate", lambda f: lambda x, n, b: f(x.flip(-1), n, b).flip(-1)),
    "turned taps": ("short_conv", lambda f: lambda x, w: f(x, w.flip(1))),
    "no past in the convolution": ("short_conv", lambda f: lambda x, w: torch.cat([f(x[:64], w), f(x[64:], w)])),
    "state lost": ("delta_rule", lambda f: lambda *a: torch.cat([f(*(x[:64] for x in a)), f(*(x[64:] for x in a))])),
    "memory lost": ("matrix_memory", lambda f: lambda *a: torch.cat([f(*(x[:64] for x in a)), f(*(x[64:] for x in a))])),
    "no decay": ("head_decay", lambda f: lambda h, t, p: torch.ones_like(f(h, t, p))),
    "no cap": ("soft_cap", lambda f: lambda x, c: x),
    "tanh gelu": ("gelu", lambda f: lambda x: torch.nn.functional.gelu(x, approximate="tanh")),
    "no groups": ("choose", lambda f: lambda c, g, n: f(c, {"count": 1, "keep": 1}, n)),
    "closed experts count as 0": ("choose", lambda f: lambda c, g, n: sorted(
        range(c.numel()), key=lambda e: -(float(c[e]) if e in f(c, g, n) else 0.0))[:n]),
    "open shared gate": ("shared_expert", lambda f: lambda h, t, p: oracle.glu(h, t, p + "shared.")),
    "no depth average": ("depth_average", lambda f: lambda xs, w: xs[-1]),
    "embedding left out": ("depth_average", lambda f: lambda xs, w: f(xs[1:], w[1:])),
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
    # the two forms of gelu are close by design
    assert ((bad - good).norm(dim=-1) / good.norm(dim=-1)).max() > \
        (1.2e-4 if fault == "tanh gelu" else 5e-3)


@pytest.mark.parametrize("change", [
    lambda c: c["layers"][0]["mixer"].update(scale=0.33),
    lambda c: c["layers"][0]["mixer"]["rot"].update(base=520.0),
    lambda c: c["layers"][1]["mixer"].update(left_scale=0.52),
    lambda c: c["layers"][1]["mixer"]["left"]["q_temp"].update(every=8),
    lambda c: c["layers"][1]["mixer"]["right"].update(gate_cap=3.2),
    lambda c: c["layers"][3]["mixer"].update(right_scale=1.05),
    lambda c: c["layers"][3]["mlp"]["router"]["groups"].update(keep=3),
    lambda c: c["norm"].update(eps=2e-3)])
def test_every_constant_is_read(cpu_rig, tmp_path, change):
    """A change of one constant moves the logits, and the engine follows."""
    cfg = json.loads(json.dumps(cpu_rig.cfg))
    change(cfg)
    toks = cpu_rig.tokens(60, 0)
    want = oracle.forward(cfg, cpu_rig.t, toks)[0]
    good = cpu_rig.logits(toks)
    assert ((want - good).norm(dim=-1) / good.norm(dim=-1)).max() > 1e-3
    other = decoder_rig.Rig(tmp_path, cfg, cpu_rig.t, oracle, "cpu")
    other.check(other.run(other.replayer(), "a", toks, [50, 1, 9]), want)


def test_closed_forms_of_the_oracle():
    """The oracle itself, where a hand can follow it."""
    one = torch.ones(1, 1, 1, dtype=D64)
    # one key of score ln 3 beside the sink: 3 / (1 + 3)
    assert math.isclose(float(oracle.attend(one, one * math.log(3), one, 1.0, None, True)), 0.75)
    # a memory's first token: v k q e^{i - m} / max(|.|, e^{-m}), m = max(f, i)
    for i, want in ((2.0, 1.0), (-3.0, math.exp(-3.0))):
        o = oracle.matrix_memory(one, one, one, torch.full((1, 1), i, dtype=D64),
                                 torch.full((1, 1), -0.5, dtype=D64))
        assert math.isclose(float(o), want, rel_tol=1e-5)
