#!/usr/bin/env python3
"""Flagship benchmark: incidents/hr end-to-end RCA (Llama-3-8B agent).

Driver contract:
    python bench.py --gpus N --steps K --warmup W
For N>1 the driver launches this under torch.distributed.run with one rank
per GPU (DP: each rank serves its own shard of concurrent investigations —
weak scaling, the reference's Celery-worker model mapped onto GPUs).

Two modes:

* ``--mode e2e`` (default, the headline): one STEP = --concurrency synthetic
  PagerDuty webhooks driven through the REAL service pipeline on this rank —
  webhook normalise/correlate -> incident row -> queue -> admission ->
  run_background_chat -> the guardrailed agent workflow (input rail, per-turn
  ToolCallGrammar-constrained action decoding, real tool execution against
  the org store / GPU RAG index, per-turn embedding-rail classification of
  tool outputs) -> forced final RCA -> summarization LLM pass ->
  recommendations -> citations -> postmortem row. The timed region contains
  ALL of it (reference pipeline: chat/background/task.py:447-697; metric
  definition BASELINE.json). p50 time-to-RCA = webhook send -> completion
  event per incident.

* ``--mode engine``: the engine-level path (per-turn RAG + rail around raw
  eng.step() decode turns) — quoted alongside for comparability.

* ``--mode layers``: prefill and decode throughput of a few full-width layers
  of a layer-listed decoder (``--design``: Kikalix beside a Mixtral-style model,
  Senotar beside a Llama-style one, Gakupel beside Kikalix, Fezuzen beside
  Gakupel) and as many of the other of equal width, heads, experts and
  feed-forward (random weights), each through its engine's own batch building,
  kernels and decode graphs, the two timed in turn.

Data: synthetic alert payloads / token streams, random-init weights
(no network in this environment).

Rank 0 prints ONE JSON line; value = whole-job incidents/hr over all ranks.
"""
from __future__ import annotations

import argparse
import asyncio
import json
import os
import statistics
import time

import torch


def parse_args():
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=2)
    ap.add_argument("--warmup", type=int, default=1)
    ap.add_argument("--mode", choices=("e2e", "engine", "layers"),
                    default=os.environ.get("BENCH_MODE", "e2e"))
    ap.add_argument("--model", default=os.environ.get("BENCH_MODEL", "llama3-8b"))
    ap.add_argument("--concurrency", type=int,
                    default=int(os.environ.get("BENCH_CONCURRENCY", "128")))
    ap.add_argument("--turns", type=int, default=int(os.environ.get("BENCH_TURNS", "4")))
    ap.add_argument("--first-prompt", type=int, default=768)
    ap.add_argument("--turn-prompt", type=int, default=512)
    ap.add_argument("--decode-per-turn", type=int, default=128)
    ap.add_argument("--device", default="auto")
    ap.add_argument("--layers", type=int, default=4,
                    help="layers per model in --mode layers")
    ap.add_argument("--size", default="all",
                    help="one of the --mode layers sizes, or all")
    ap.add_argument("--design", choices=("kikalix", "senotar", "gakupel", "fezuzen"),
                    default="kikalix",
                    help="design of --mode layers")
    ap.add_argument("--rag", type=int, default=int(os.environ.get("BENCH_RAG", "1")),
                    help="per-turn on-GPU RAG retrieval + input-rail check (1=on)")
    ap.add_argument("--rag-docs", type=int,
                    default=int(os.environ.get("BENCH_RAG_DOCS", "10000")))
    return ap.parse_args()


def synth_tokens(rng: torch.Generator, n: int, vocab: int) -> list:
    return torch.randint(0, min(vocab - 4, 250), (n,), generator=rng).tolist()


# --------------------------------------------------------------------------
# engine mode (comparability path)
# --------------------------------------------------------------------------

class RagPath:
    """Engine mode: per-turn retrieval over an HBM-resident corpus
    (on-GPU sentence encoder + kNN) + the input-rail heuristic check."""

    def __init__(self, args, device: str):
        import torch as _t
        from aurora_amd import ops
        from aurora_amd.models.encoder import SentenceEncoder
        self.ops = ops
        self.device = device
        self.encoder = SentenceEncoder(
            "bge-base", dtype=_t.bfloat16 if device != "cpu" else _t.float32,
            device=device)
        self.encoder.init_random(3)
        rng = _t.Generator().manual_seed(17)
        chunks = [_t.randint(1, 250, (96,), generator=rng).tolist()
                  for _ in range(args.rag_docs)]
        embs = []
        for i in range(0, len(chunks), 512):
            embs.append(self.encoder.encode_ids(chunks[i:i + 512]))
        self.docs = _t.cat(embs)
        self.rail_patterns = None

    def rail_check(self, tokens) -> bool:
        from aurora_amd.guardrails.input_rail import _INJECTION_PATTERNS
        text = bytes(t % 256 for t in tokens[:512]).decode("latin-1")
        return not any(p.search(text) for p in _INJECTION_PATTERNS)

    def retrieve(self, query_tokens) -> list:
        qv = self.encoder.encode_ids([query_tokens[:96]])
        vals, idx = self.ops.knn_topk(qv, self.docs, 4)
        out = []
        for i in idx[0].tolist():
            out.extend(((i * 131 + j * 7) % 250 for j in range(32)))
        return out


def run_step_engine(eng, args, rng, vocab, step_idx: int, rag=None):
    """One engine-level investigation batch; returns per-incident latencies."""
    from aurora_amd.engine.sampling_params import SamplingParams

    B, turns = args.concurrency, args.turns
    params = SamplingParams(temperature=0.7, top_p=0.95,
                            max_tokens=args.decode_per_turn, ignore_eos=True)
    ctx_tokens = {i: synth_tokens(rng, args.first_prompt, vocab) for i in range(B)}
    turn_no = {i: 0 for i in range(B)}
    t_start = {i: time.monotonic() for i in range(B)}
    t_done = {}

    def submit(i):
        rid = f"s{step_idx}-inc{i}-t{turn_no[i]}"
        if rag is not None:
            rag.rail_check(ctx_tokens[i][-args.turn_prompt:])
            retrieved = rag.retrieve(ctx_tokens[i][-96:])
            ctx_tokens[i][-len(retrieved):] = retrieved  # fixed token count
        eng.add_request(rid, list(ctx_tokens[i]), params, session_id=f"inc-{step_idx}-{i}")
        return rid

    live = {}
    for i in range(B):
        live[submit(i)] = i
    gen_out = {i: [] for i in range(B)}
    while live:
        for out in eng.step():
            i = live.get(out.request_id)
            if i is None:
                continue
            gen_out[i].extend(out.new_token_ids)
            if out.finished:
                del live[out.request_id]
                ctx_tokens[i].extend(gen_out[i][-args.decode_per_turn:])
                turn_no[i] += 1
                if turn_no[i] < turns:
                    ctx_tokens[i].extend(synth_tokens(rng, args.turn_prompt, vocab))
                    live[submit(i)] = i
                else:
                    t_done[i] = time.monotonic()
    return [t_done[i] - t_start[i] for i in range(B)]


def main_engine(args, rank, world, use_cuda):
    from aurora_amd.engine.engine import EngineConfig, LLMEngine
    from aurora_amd.models.config import get_spec
    from aurora_amd.parallel import dist as pdist

    spec = get_spec(args.model)
    cfg = EngineConfig(
        model=args.model,
        device="cpu" if not use_cuda else "auto",
        max_num_seqs=max(args.concurrency + 2, 8),
        max_batched_tokens=16384,
        seed=1234 + rank,
    )
    eng = LLMEngine(cfg)
    rng = torch.Generator().manual_seed(999 + rank)
    vocab = spec.vocab_size
    rag = RagPath(args, eng.device) if args.rag else None

    def sync():
        if use_cuda:
            torch.cuda.synchronize()
        if world > 1:
            pdist.barrier()
            if use_cuda:
                torch.cuda.synchronize()

    for w in range(args.warmup):
        run_step_engine(eng, args, rng, vocab, -1 - w, rag)
    sync()
    t0 = time.monotonic()
    lat = []
    for s in range(args.steps):
        lat.extend(run_step_engine(eng, args, rng, vocab, s, rag))
    sync()
    elapsed = time.monotonic() - t0
    extra = {
        "pipeline": "engine",
        "rag": bool(rag), "rag_docs": args.rag_docs if rag else 0,
        "guardrail_per_turn": bool(rag),
        "decode_tokens_per_turn": args.decode_per_turn,
        "prompt_tokens_per_incident": args.first_prompt
        + (args.turns - 1) * args.turn_prompt,
        "engine_timers_s": {k: round(v, 2) for k, v in eng.timers.items()},
        "engine_counters": eng.counters,
    }
    return elapsed, lat, extra


# --------------------------------------------------------------------------
# e2e mode (the headline): real webhook -> worker -> workflow -> summary
# --------------------------------------------------------------------------

#: fast read-only tools the random-weight agent may call during the bench —
#: real registry tools hitting the org store / infra graph / GPU RAG
#: ("stub-fast" tool execution per the metric definition; exec-style tools
#: are excluded so a random-weight model can't run shell commands)
BENCH_TOOLS = [
    "knowledge_base_search", "list_incidents", "get_incident",
    "get_incident_timeline", "get_alert_field", "list_services",
    "get_service_impact", "get_infrastructure_context", "final_answer",
]

_LOREM = ("deploy rollout canary latency p99 spike postgres connection pool "
          "exhausted kafka lag consumer rebalance oom killed node pressure "
          "dns resolution timeout ingress 502 upstream retry storm cache "
          "eviction hot shard gc pause tls handshake certificate expired").split()


def _synth_doc(rng: torch.Generator, n_words: int = 160) -> str:
    idx = torch.randint(0, len(_LOREM), (n_words,), generator=rng).tolist()
    return " ".join(_LOREM[i] for i in idx)


def _build_runtime(args, rank, use_cuda):
    os.environ.setdefault("AURORA_RAIL_BACKEND", "encoder")
    from aurora_amd.engine.engine import EngineConfig
    from aurora_amd.engine.server import AsyncEngineServer
    from aurora_amd.service.runtime import Runtime
    from aurora_amd.utils.config import Settings

    scfg = Settings(db_path=":memory:",
                    secrets_path=f"/tmp/bench_secrets_{rank}.json")
    scfg.worker_concurrency = args.concurrency + 8
    scfg.max_concurrent_rca = args.concurrency * 2
    scfg.rca_max_turns = args.turns
    scfg.guardrails_enabled = True
    ecfg = EngineConfig(
        model=args.model,
        device="cpu" if not use_cuda else "auto",
        max_num_seqs=max(args.concurrency + 2, 8),
        max_batched_tokens=16384,
        kv_memory_fraction=float(os.environ.get("KV_MEMORY_FRACTION", "0.8")),
        seed=1234 + rank,
    )
    server = AsyncEngineServer(ecfg)
    rt = Runtime(scfg, engine_server=server)
    org_id = rt.admin.create_org(f"bench-{rank}")
    rt.admin.create_user(org_id, f"bench{rank}@aurora.local",
                         user_id=f"bench-user-{rank}")
    # infra graph for the graph tools
    g = rt.graph(org_id)
    for svc in ("api", "db", "cache", "queue", "ingress"):
        g.upsert_service(svc)
    for a, b in (("api", "db"), ("api", "cache"), ("ingress", "api"),
                 ("queue", "db")):
        g.add_dependency(a, b)
    # RAG corpus: args.rag_docs synthetic chunks embedded on the GPU encoder
    # (HBM-resident kNN bank) without round-tripping SQLite at bench setup
    rag = rt.rag(org_id)
    rng = torch.Generator().manual_seed(17)
    docs = [_synth_doc(rng) for _ in range(args.rag_docs)]
    BATCH = 512
    for i in range(0, len(docs), BATCH):
        batch = docs[i:i + BATCH]
        vecs = rag._embed(batch)
        for j, d in enumerate(batch):
            rag.chunks.append({"text": d, "doc_id": f"kb-{i + j}",
                               "doc_name": f"runbook-{(i + j) % 97}"})
            rag.bm25.add(d)
        if vecs is not None:
            vecs = vecs.to(rag.device)
            rag.emb = vecs if rag.emb is None else torch.cat([rag.emb, vecs])
    return rt, org_id


def _payload(rng: torch.Generator, step: int, i: int) -> dict:
    """Unique synthetic PagerDuty v3 event. Every alert must open a NEW
    incident, so its text is made lexically unique (the correlator's
    similarity strategy would otherwise merge same-vocabulary alerts —
    which is correct behavior for real alert storms)."""
    tag = f"s{step}i{i}"
    doc = " ".join(f"{w}{tag}" for w in _synth_doc(rng, 60).split())
    return {"event": {"data": {
        "id": f"PD-{step}-{i}-{torch.randint(0, 1 << 30, (1,), generator=rng).item()}",
        "title": f"[bench s{step}] {doc[:80]} #{i}",
        "service": {"summary": f"svc-{step}-{i}"},
        "priority": {"summary": "P2"},
        "urgency": "high",
        "body": {"details": doc},
    }}}


async def run_step_e2e(rt, org_id, args, rng, step: int,
                       deadline_s: float = 1500.0):
    import sys
    from aurora_amd.service.webhooks import process_webhook
    B = args.concurrency
    ev_q = rt.events.subscribe(org_id)
    t_start: dict = {}
    pending = set()
    statuses: dict = {}
    t0 = time.monotonic()
    for i in range(B):
        t_start_i = time.monotonic()
        iid, created = process_webhook(
            rt, org_id, "pagerduty", _payload(rng, step, i),
            rca_countdown_s=0.0,
            rca_args={"max_turns": args.turns, "tool_subset": BENCH_TOOLS})
        assert created, f"correlator merged bench alert {i} into {iid}"
        t_start[iid] = t_start_i
        pending.add(iid)
    lat = []
    last_beat = t0
    while pending:
        left = deadline_s - (time.monotonic() - t0)
        if left <= 0:
            # stragglers the deadline cut off: reported, and EXCLUDED from
            # the throughput numerator (work the timed region didn't finish)
            print(f"[bench] step {step}: deadline, {len(pending)} pending",
                  file=sys.stderr, flush=True)
            statuses["straggler"] = statuses.get("straggler", 0) + len(pending)
            break
        try:
            ev = await asyncio.wait_for(ev_q.get(), timeout=min(left, 30.0))
        except asyncio.TimeoutError:
            ev = None
        now = time.monotonic()
        if now - last_beat > 30.0:
            last_beat = now
            c = rt.engine.engine.counters
            print(f"[bench] step {step} t={now - t0:.0f}s done="
                  f"{len(lat)}/{B} counters={c}", file=sys.stderr, flush=True)
        if (ev and ev.get("type") == "incident_update"
                and ev.get("incident_id") in pending
                and ev.get("aurora_status") in ("completed", "failed")):
            iid = ev["incident_id"]
            pending.discard(iid)
            statuses[ev["aurora_status"]] = statuses.get(ev["aurora_status"], 0) + 1
            lat.append(time.monotonic() - t_start[iid])
    rt.events.unsubscribe(org_id, ev_q)
    return lat, statuses


async def main_e2e_async(args, rank, world, use_cuda):
    from aurora_amd.parallel import dist as pdist

    rt, org_id = _build_runtime(args, rank, use_cuda)
    rt.start()
    rng = torch.Generator().manual_seed(999 + rank)

    def sync():
        if use_cuda:
            torch.cuda.synchronize()
        if world > 1:
            pdist.barrier()
            if use_cuda:
                torch.cuda.synchronize()

    statuses_all: dict = {}
    for w in range(args.warmup):
        await run_step_e2e(rt, org_id, args, rng, -1 - w)
    sync()
    t0 = time.monotonic()
    lat = []
    for s in range(args.steps):
        l, st = await run_step_e2e(rt, org_id, args, rng, s)
        lat.extend(l)
        for k, v in st.items():
            statuses_all[k] = statuses_all.get(k, 0) + v
    sync()
    elapsed = time.monotonic() - t0

    eng = rt.engine.engine
    extra = {
        "pipeline": "webhook->queue->workflow->summary (end-to-end)",
        "in_timed_region": ["webhook normalise+correlate", "queue dispatch",
                           "input rail", "per-turn grammar tool decode",
                           "tool execution", "per-turn tool-output rail",
                           "GPU RAG (kb tool)", "forced final RCA",
                           "summarization pass", "recommendations",
                           "citations", "postmortem"],
        "rag_docs": args.rag_docs,
        "guardrail_per_turn": True,
        "tool_subset": BENCH_TOOLS,
        "completed": statuses_all.get("completed", 0),
        "failed_terminal": statuses_all.get("failed", 0),
        "stragglers": statuses_all.get("straggler", 0),
        "engine_timers_s": {k: round(v, 2) for k, v in eng.timers.items()},
        "engine_counters": eng.counters,
    }
    await rt.stop()
    rt.engine.shutdown()
    return elapsed, lat, extra


# --------------------------------------------------------------------------
# layers mode: a design's layers beside the closest model's of equal size
# --------------------------------------------------------------------------

#: width, heads, kv heads, experts, top, ff: layers of a 7B-class decoder with
#: few wide experts, of one with many narrow experts, and of a small one
LAYER_SIZES = {
    "4096-8x14336": (4096, 32, 8, 8, 2, 14336),
    "2048-64x1408": (2048, 16, 8, 64, 6, 1408),
    "1024-16x512": (1024, 8, 2, 16, 2, 512),
}
#: width, heads, kv heads of the Llama-style layers, latent rank, ff
SENOTAR_SIZES = {
    "4096-14336": (4096, 32, 8, 512, 14336),
    "2048-5632": (2048, 16, 4, 512, 5632),
    "1024-2816": (1024, 16, 4, 256, 2816),
}
#: width, heads, kv heads, experts, top, expert ff, shared ff, dense ff
GAKUPEL_SIZES = {
    "4096-8x14336": (4096, 32, 8, 8, 2, 14336, 3584, 14336),
    "2048-64x1408": (2048, 16, 4, 64, 6, 1408, 2816, 5632),
    "1024-16x512": (1024, 8, 2, 16, 2, 512, 1024, 2816),
}
#: width, heads, kv heads, latent rank, queries' rank, unrotated and rotated width of a
#: latent-attention head, experts, top, expert ff, shared ff
FEZUZEN_SIZES = {
    "4096-8x14336": (4096, 32, 8, 512, 1536, 128, 64, 8, 2, 14336, 3584),
    "2048-64x1408": (2048, 16, 4, 512, 1024, 128, 64, 64, 6, 1408, 2816),
    "1024-16x512": (1024, 8, 2, 256, 512, 64, 32, 16, 2, 512, 1024),
}
PREFILL_SEQS, PREFILL_LEN, DECODE_SEQS, DECODE_STEPS = 4, 2048, 64, 32


def layer_pair(size: str, n_layers: int):
    """(Kikalix spec, Mixtral-style spec) of one size."""
    from aurora_amd.models.config import HybridSpec, ModelSpec, kikalix_layers
    w, h, kv, experts, top, ff = LAYER_SIZES[size]
    d = w // h
    pattern = ("pppr" * n_layers)[:n_layers]
    hybrid = HybridSpec(
        name=f"kikalix-{size}", hidden_size=w, vocab_size=32000, max_position=8192,
        layers=kikalix_layers(
            pattern, heads=h, kv_heads=kv, dim=d, vdim=d, window=1024, d_heads=h // 2,
            d_kv_heads=h // 2, d_dim=d, d_vdim=d, rank=128, r_heads=h // 2, r_dim=d,
            r_vdim=2 * d, experts=experts, top=top, ff=ff))
    mixtral = ModelSpec(
        name=f"mixtral-{size}", hidden_size=w, n_layers=n_layers, n_heads=h, n_kv_heads=kv,
        head_dim=d, intermediate_size=ff, vocab_size=32000, max_position=8192,
        n_experts=experts, experts_per_token=top)
    return hybrid, mixtral


def senotar_pair(size: str, n_layers: int):
    """(Senotar spec, Llama-style spec) of one size; every second Senotar layer
    reads the latents of the one before it."""
    from aurora_amd.models.config import ModelSpec, senotar_spec
    w, h, kv, rank, ff = SENOTAR_SIZES[size]
    d = w // h
    senotar = senotar_spec(
        f"senotar-{size}", ("os" * n_layers)[:n_layers], width=w, vocab=32000, heads=h,
        dim=d, vdim=d, kv_rank=rank, ff=ff, max_position=8192)
    llama = ModelSpec(
        name=f"llama-{size}", hidden_size=w, n_layers=n_layers, n_heads=h, n_kv_heads=kv,
        head_dim=d, intermediate_size=ff, vocab_size=32000, max_position=8192)
    return senotar, llama


def gakupel_pair(size: str, n_layers: int):
    """(Gakupel spec, Kikalix spec without a window) of one size: a recurrence in as
    many layers, experts in as many as have them, heads and states of equal size."""
    from aurora_amd.models.config import HybridSpec, gakupel_spec, kikalix_layers
    w, h, kv, experts, top, ff, shared, dense = GAKUPEL_SIZES[size]
    d = w // h
    gakupel = gakupel_spec(
        f"gakupel-{size}", ("pdaP" * n_layers)[:n_layers], width=w, vocab=32000, heads=h,
        kv_heads=kv, dim=d, l_dim=d, l_vdim=d, d_heads=h // 2, d_kv_heads=h // 2, d_dim=d,
        d_vdim=d, m_heads=h // 2, m_dim=d, m_vdim=2 * d, ff=dense, experts=experts, top=top,
        expert_ff=ff, shared_ff=shared, groups=4, keep=2, max_position=8192)
    kikalix = HybridSpec(
        name=f"kikalix-{size}", hidden_size=w, vocab_size=32000, max_position=8192,
        layers=kikalix_layers(
            ("pppr" * n_layers)[:n_layers], heads=h, kv_heads=kv, dim=d, vdim=d, window=0,
            d_heads=h // 2, d_kv_heads=h // 2, d_dim=d, d_vdim=d, rank=128, r_heads=h // 2,
            r_dim=d, r_vdim=2 * d, experts=experts, top=top, ff=ff))
    return gakupel, kikalix


def fezuzen_pair(size: str, n_layers: int):
    """(Fezuzen spec, Gakupel spec) of one size: windows of half a prompt and chunks of
    three quarters, every second latent layer borrowing, beside full attention; routed
    experts and a shared one in every layer of both."""
    from aurora_amd.models.config import fezuzen_spec, gakupel_spec
    w, h, kv, rank, q_rank, dim, rot, experts, top, ff, shared = FEZUZEN_SIZES[size]
    d = w // h
    fezuzen = fezuzen_spec(
        f"fezuzen-{size}", ("oasa" * n_layers)[:n_layers], width=w, vocab=32000, heads=h,
        dim=dim, rot_dim=rot, vdim=dim, kv_rank=rank, q_rank=q_rank, window=1024, a_heads=h,
        kv_heads=kv, a_dim=d, a_vdim=d, chunk=1536, experts=experts, top=top, expert_ff=ff,
        shared_ff=shared, groups=4, keep=2, max_position=8192)
    gakupel = gakupel_spec(
        f"gakupel-{size}", "a" * n_layers, width=w, vocab=32000, heads=h,
        kv_heads=kv, dim=d, l_dim=d, l_vdim=d, d_heads=h, d_kv_heads=h, d_dim=d, d_vdim=d,
        m_heads=h, m_dim=d, m_vdim=d, ff=ff, experts=experts, top=top, expert_ff=ff,
        shared_ff=shared, groups=4, keep=2, max_position=8192)
    return fezuzen, gakupel


def layer_bench_engine(spec, seed: int = 0):
    from aurora_amd.engine.engine import EngineConfig, LLMEngine
    from aurora_amd.models.registry import build_model
    cuda = torch.cuda.is_available()
    model = build_model(spec, torch.bfloat16 if cuda else torch.float32,
                        "cuda" if cuda else "cpu", seed=seed)
    return LLMEngine(EngineConfig(
        model=spec.name, max_num_seqs=DECODE_SEQS, state_slots=DECODE_SEQS, max_model_len=4096,
        kv_cache_pages=DECODE_SEQS * 16 + 1, page_size=256, prefix_cache=False), model=model)


def layer_bench_once(eng, rng):
    """(prefill seconds, decode seconds per step) of one timed pass."""
    from aurora_amd.engine.engine import Sequence
    from aurora_amd.engine.sampling_params import SamplingParams

    def fresh(n):
        seqs = []
        for i in range(n):
            s = Sequence(f"b{i}", synth_tokens(rng, PREFILL_LEN, eng.spec.vocab_size),
                         SamplingParams())
            assert eng._try_reserve(s, PREFILL_LEN + DECODE_STEPS + 1)
            seqs.append(s)
        return seqs

    seqs = fresh(DECODE_SEQS)
    waves = [seqs[i:i + PREFILL_SEQS] for i in range(0, DECODE_SEQS, PREFILL_SEQS)]
    t0 = time.monotonic()
    for wave in waves:
        eng.execute(wave, [PREFILL_LEN] * len(wave), [],
                    [PREFILL_LEN * (i + 1) - 1 for i in range(len(wave))])
    t1 = time.monotonic()
    for _ in range(DECODE_STEPS):
        for s in seqs:
            s.token_ids.append(7)
        eng.execute([], [], seqs, list(range(len(seqs))))
    t2 = time.monotonic()
    for s in seqs:
        eng._release(s)
    return t1 - t0, (t2 - t1) / DECODE_STEPS


def main_layers(args):
    table, pair = {"kikalix": (LAYER_SIZES, layer_pair),
                   "senotar": (SENOTAR_SIZES, senotar_pair),
                   "gakupel": (GAKUPEL_SIZES, gakupel_pair),
                   "fezuzen": (FEZUZEN_SIZES, fezuzen_pair)}[args.design]
    sizes = list(table) if args.size == "all" else [args.size]
    result = {}
    for size in sizes:
        engines = {s.name.split("-")[0]: layer_bench_engine(s)
                   for s in pair(size, args.layers)}
        rng = torch.Generator().manual_seed(5)
        best = {k: [float("inf"), float("inf")] for k in engines}
        for it in range(args.warmup + args.steps):
            for k, eng in engines.items():  # in turn
                pre, dec = layer_bench_once(eng, rng)
                if it >= args.warmup:
                    best[k] = [min(best[k][0], pre), min(best[k][1], dec)]
        tokens = DECODE_SEQS * PREFILL_LEN
        result[size] = {k: {"prefill_tok_s": round(tokens / p),
                            "decode_tok_s": round(DECODE_SEQS / d),
                            "decode_ms_per_step": round(d * 1e3, 3)}
                        for k, (p, d) in best.items()}
        del engines, eng
        if torch.cuda.is_available():
            torch.cuda.empty_cache()
    print(json.dumps({
        "metric": "tokens/s", "mode": "layers", "layers": args.layers,
        "prefill": f"{PREFILL_SEQS} x {PREFILL_LEN} tokens per batch",
        "decode": f"{DECODE_SEQS} sequences at {PREFILL_LEN} tokens",
        "dtype": "bf16", "data": "synthetic", "sizes": result}))


def main():
    args = parse_args()
    if args.mode == "layers":
        main_layers(args)
        return
    rank = int(os.environ.get("RANK", "0"))
    world = int(os.environ.get("WORLD_SIZE", "1"))
    use_cuda = torch.cuda.is_available() and args.device != "cpu"

    from aurora_amd.parallel import dist as pdist
    if world > 1:
        pdist.init_distributed(tp_size=1)

    if args.mode == "engine":
        elapsed, lat, extra = main_engine(args, rank, world, use_cuda)
    else:
        elapsed, lat, extra = asyncio.run(
            main_e2e_async(args, rank, world, use_cuda))

    # incidents that reached a terminal status inside the deadline; in
    # engine mode every submitted incident completes by construction.
    # Stragglers cut off by the e2e deadline must NOT count in the
    # numerator — that would credit work the timed region didn't finish.
    done_local = float(extra.get("completed", 0) + extra.get("failed_terminal", 0)
                       if args.mode == "e2e"
                       else args.steps * args.concurrency)

    # max over ranks (slowest rank defines the job); sum of terminal counts
    if world > 1:
        import torch.distributed as dist
        dev = "cuda" if (use_cuda and dist.get_backend() == "nccl") else "cpu"
        t = torch.tensor([elapsed], device=dev)  # RCCL needs device tensors
        dist.all_reduce(t, op=dist.ReduceOp.MAX)
        elapsed = float(t[0])
        d = torch.tensor([done_local], device=dev)
        dist.all_reduce(d, op=dist.ReduceOp.SUM)
        incidents = int(d[0])
    else:
        incidents = int(done_local)
    value = incidents / (elapsed / 3600.0)
    p50 = statistics.median(lat) if lat else 0.0
    tokens_per_incident = (args.first_prompt + (args.turns - 1) * args.turn_prompt
                           + args.turns * args.decode_per_turn)
    if rank == 0:
        print(json.dumps({
            "metric": "incidents/hr",
            "value": round(value, 2),
            "unit": "incidents/hr",
            "n_gpus": world if use_cuda else 0,
            "steps": args.steps,
            "warmup": args.warmup,
            "ms_per_step": round(elapsed / args.steps * 1000.0, 2),
            "higher_is_better": True,
            "scaling": "weak",
            "vs_baseline": None,
            "dtype": "bf16" if use_cuda else "fp32",
            "data": "synthetic",
            "config": {
                "model": args.model,
                "mode": args.mode,
                "global_batch": args.concurrency * world,
                "seq_len": tokens_per_incident,
                "parallelism": f"dp{world}",
                "concurrency_per_gpu": args.concurrency,
                "turns": args.turns,
                "p50_time_to_rca_s": round(p50, 3),
                **extra,
            },
        }))


if __name__ == "__main__":
    main()
