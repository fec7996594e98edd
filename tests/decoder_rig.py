"""A checkpoint on disk, its plain oracle, and engines over it: what the tests of
every layer-listed design share."""
import json
import os

import torch
from safetensors.torch import save_file

from aurora_amd.engine.engine import EngineConfig, LLMEngine
from aurora_amd.engine.replay import TraceReplayer, make_engine
from aurora_amd.engine.sampling_params import SamplingParams


class Rig:
    def __init__(self, path, cfg, tensors, oracle, device, dtype="float32", bf16_tol=0.1):
        self.bf16_tol = bf16_tol
        self.cfg, self.t, self.oracle = cfg, tensors, oracle
        self.device, self.dtype = device, dtype
        self.path = str(path)
        with open(os.path.join(self.path, "config.json"), "w") as f:
            json.dump(self.cfg, f)
        save_file(self.t, os.path.join(self.path, "model.safetensors"))
        self._logits = {}

    def tokens(self, n, seed):
        gen = torch.Generator().manual_seed(100 + seed)
        return torch.randint(0, self.cfg["vocab"], (n,), generator=gen).tolist()

    def logits(self, toks):
        key = tuple(toks)
        if key not in self._logits:
            self._logits[key] = self.oracle.forward(self.cfg, self.t, toks)[0]
        return self._logits[key]

    def replayer(self, max_tokens=1024, page=16, requests=4):
        return TraceReplayer(make_engine(self.path, self.dtype, max_tokens, self.device,
                                         requests, page))

    def engine(self, **kw):
        return LLMEngine(EngineConfig(model=self.path, dtype=self.dtype, device=self.device,
                                      **{"page_size": 16, **kw}))

    def check(self, got, want, tol=None):
        """Every row's relative error."""
        tol = tol or (1e-4 if self.dtype == "float32" else self.bf16_tol)
        got, want = got.double().cpu(), want.double()
        err = (got - want).norm(dim=-1) / want.norm(dim=-1)
        assert err.max() < tol, [round(float(e), 5)
                                 for e in err.sort(descending=True).values[:20]]

    def run(self, rp, rid, toks, cuts):
        """Logits of every token of a request fed in portions of ``cuts``."""
        out, at = [], 0
        for c in cuts:
            out.append(rp.step([(rid, toks[at:at + c], list(range(c)))]).cpu())
            at += c
        assert at == len(toks)
        rp.step([], [rid])
        return torch.cat(out)

    def run_plan(self, rp, toks, plan):
        """Feed steps of {request: number of its next tokens}; every request's
        logits against its own as if it were alone."""
        at, got = dict.fromkeys(toks, 0), {r: [] for r in toks}
        for step in plan:
            entries = [(r, toks[r][at[r]:at[r] + n], list(range(n))) for r, n in step.items()]
            for r, n in step.items():
                at[r] += n
            rows = rp.step(entries, [r for r in step if at[r] == len(toks[r])]).cpu()
            for r, n in step.items():
                got[r].append(rows[:n])
                rows = rows[n:]
        for r in toks:
            self.check(torch.cat(got[r]), self.logits(toks[r]))
        assert not rp.live

    def trail(self, toks):
        """The residual stream after every layer run of one prompt."""
        rp, trail = self.replayer(), []
        model = rp.engine.model
        forward = model.forward
        model.forward = lambda *a: forward(*a, trail=trail)
        try:
            rp.step([("a", toks, [0])])
        finally:
            model.forward = forward
        return trail

    def check_greedy(self, prompts, outs, n):
        """The chosen token's oracle logit is the highest, up to rounding."""
        for p, got in zip(prompts, outs):
            assert len(got) == n
            lg = self.logits(p + got)[len(p) - 1:-1]
            gap = lg.max(-1).values - lg[torch.arange(n), torch.tensor(got)]
            assert gap.max() < (1e-3 if self.dtype == "float32" else 0.35), gap

    def greedy(self, prompt, n):
        toks = list(prompt)
        for _ in range(n):
            toks.append(int(self.oracle.forward(self.cfg, self.t, toks)[0][-1].argmax()))
        return toks[len(prompt):]


GREEDY = dict(temperature=0.0, ignore_eos=True)


def turn(eng, rid, toks, n, session=None):
    """One greedy request driven to its end; its new tokens."""
    eng.add_request(rid, toks, SamplingParams(max_tokens=n, **GREEDY), session_id=session)
    out = []
    while eng.has_work():
        for o in eng.step():
            out += o.new_token_ids
    return out
