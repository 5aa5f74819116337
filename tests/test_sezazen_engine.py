"""Sezazen in the engine: every way of cutting and batching a sequence against
the plain whole-sequence oracle, on the CPU ops and on the HIP kernels."""
import copy
import io
import itertools
import json
import os
import subprocess
import sys

import pytest
import torch

import sezazen_models as M
import sezazen_oracle as oracle
from engine_helpers import close, feed, worker
from llm_d_inference_scheduler_amd import trace
from llm_d_inference_scheduler_amd.engine import EngineRequest, EngineWorker
from llm_d_inference_scheduler_amd.engine.worker import TokenSpan
from llm_d_inference_scheduler_amd.models import registry, sezazen

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
GPU = pytest.mark.gpu
# (device, dtype, tolerance on the rms error relative to the logits' rms, mean
# over the tokens)
RUNS = [pytest.param(("cpu", torch.float32, 1e-5), id="cpu-f32"),
        pytest.param(("cuda:0", torch.float32, 1e-5), id="gpu-f32",
                     marks=GPU),
        pytest.param(("cuda:0", torch.bfloat16, 3e-2), id="gpu-bf16",
                     marks=GPU)]
CPU = ("cpu", torch.float32, 1e-5)
CONFIGS = {"odd": M.ODD, "tiled": M.TILED, "once": M.ONCE,
           "straight": M.STRAIGHT}


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    """name -> (folder, config, weights), and oracle logits by tokens."""
    made, known = {}, {}

    def get(name, cfg=None, weights=None):
        if name not in made:
            cfg = cfg or CONFIGS[name]
            folder, w = M.write_model(
                tmp_path_factory.mktemp(name), cfg, weights, seed=len(name))
            made[name] = (folder, cfg, w)
        return made[name]

    def expect(name, toks):
        key = (name, tuple(toks))
        if key not in known:
            _, cfg, w = made[name]
            known[key] = oracle.forward(cfg, w, toks)
        return known[key]
    get.expect = expect
    return get


def generate(w, prompts, max_tokens):
    """Through add_request/step -> {request: generated tokens}."""
    for rid, p in prompts.items():
        w.add_request(EngineRequest(rid, list(p), max_tokens=max_tokens))
    done = {}
    for _ in range(300):
        for o in w.step():
            if o.finished:
                assert not o.error, o.error
                done[o.request_id] = o
        if not w.has_work:
            break
    assert set(done) == set(prompts)
    return done


def best_by_oracle(cfg, weights, prompt, made, limit):
    """Every generated token is the oracle's best, or as good as it."""
    logits = oracle.forward(cfg, weights, prompt + made)
    for i, t in enumerate(made):
        row = logits[len(prompt) - 1 + i]
        assert float(row.max() - row[t]) <= \
            8 * limit * float(row.pow(2).mean().sqrt()), i


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("name", list(CONFIGS))
class TestAgainstOracle:
    def test_whole_and_layers(self, models, name, run):
        folder, cfg, weights = models(name)
        toks = M.tokens(cfg, 150)
        want = []
        logits = oracle.forward(cfg, weights, toks, want)
        w = worker(folder, run)
        got = []
        out = w.forward_spans([TokenSpan("a", toks, list(range(150)))],
                              layers_out=got)
        assert len(got) == len(want)    # a looped layer counts every time
        for i, (a, b) in enumerate(zip(got, want)):
            close(a, b, run[2], f"run {i}")
        close(out, logits, run[2])

    def test_token_by_token(self, models, name, run):
        folder, cfg, _ = models(name)
        toks = M.tokens(cfg, 90, 1)
        w = worker(folder, run)
        close(feed(w, "a", toks, [1] * 90), models.expect(name, toks), run[2])

    @pytest.mark.parametrize("size", [2, 3, 8, 9, 16, 17, 43, 64])
    def test_portions(self, models, name, run, size):
        folder, cfg, _ = models(name)
        toks = M.tokens(cfg, 140, 2)
        cuts = [size] * (140 // size) + [140 % size] * (140 % size > 0)
        w = worker(folder, run)
        close(feed(w, "a", toks, cuts), models.expect(name, toks), run[2])

    def test_changing_portions_and_long_decoding(self, models, name, run):
        folder, cfg, _ = models(name)
        toks = M.tokens(cfg, 200, 3)
        cuts = [5, 1, 70, 2, 1, 1, 19, 12, 1, 8] + [1] * 80
        w = worker(folder, run)
        close(feed(w, "a", toks, cuts), models.expect(name, toks), run[2])

    def test_first_tokens(self, models, name, run):
        """Where the sink takes most of the weight."""
        folder, cfg, _ = models(name)
        w = worker(folder, run)
        for n, cuts in ((1, [1]), (2, [2]), (3, [1, 2]), (4, [2, 2])):
            toks = M.tokens(cfg, n, 40 + n)
            close(feed(w, f"r{n}", toks, cuts), models.expect(name, toks),
                  run[2])
            w.finish_spans(f"r{n}")

    def test_mixed_batch_equals_alone(self, models, name, run):
        """Unequal requests side by side: long and short portions, single
        tokens, one left out of some steps; pages come from freed requests."""
        folder, cfg, _ = models(name)
        w = worker(folder, run, blocks=32)
        for i in range(5):          # dirty every page first
            feed(w, f"old{i}", M.tokens(cfg, 100, 60 + i), [37, 63], False)
            w.finish_spans(f"old{i}")
        toks = {r: M.tokens(cfg, n, 70 + n) for r, n in
                (("a", 160), ("b", 45), ("c", 21), ("d", 100), ("e", 75))}
        plans = {"a": itertools.chain([90, 3, 30], itertools.repeat(1)),
                 "b": itertools.chain([9, 1, 2], itertools.repeat(1)),
                 "c": itertools.repeat(1),
                 "d": itertools.chain([1, 2, 70], itertools.repeat(3)),
                 "e": itertools.repeat(11)}
        at, got, live, step = {}, {}, ["a", "b", "c", "d"], 0
        queue = ["e"]
        while live:
            spans = []
            for r in live:
                if (step + ord(r)) % 5 == 4:
                    continue        # not in this step
                lo = at.get(r, 0)
                n = min(next(plans[r]), len(toks[r]) - lo)
                spans.append(TokenSpan(r, toks[r][lo:lo + n],
                                       list(range(n))))
                at[r] = lo + n
            if spans:
                out = w.forward_spans(spans)
                for s in spans:
                    got.setdefault(s.request_id, []).append(
                        out[:len(s.tokens)])
                    out = out[len(s.tokens):]
            for r in list(live):
                if at.get(r) == len(toks[r]):
                    live.remove(r)
                    w.finish_spans(r)
                    if queue:
                        live.append(queue.pop())
            step += 1
        for r, parts in got.items():
            close(torch.cat(parts), models.expect(name, toks[r]), run[2], r)
        assert w.mgr.free_blocks == 32

    def test_greedy_generation(self, models, name, run):
        """Admission, portions of prompts beside decoding, more requests than
        the pool holds at a time."""
        folder, cfg, weights = models(name)
        w = worker(folder, run, blocks=10, prefill_chunk_tokens=24,
                   prefill_min_tokens=1, max_decode_batch=4)
        prompts = {f"g{i}": M.tokens(cfg, n, 80 + i)
                   for i, n in enumerate((30, 1, 57, 12, 44))}
        for rid, o in generate(w, prompts, 6).items():
            assert len(o.all_tokens) == 6
            best_by_oracle(cfg, weights, prompts[rid], o.all_tokens, run[2])
        assert w.mgr.free_blocks == 10


@pytest.mark.parametrize("run", RUNS[:2])
def test_any_route(models, run):
    """Routers that read the whole stream (exact runs: rounding may turn a
    close choice)."""
    folder, cfg, _ = models("any-route", M.TILED, M.random_weights(
        M.TILED, 3, clear_routes=False))
    toks = M.tokens(cfg, 120, 4)
    w = worker(folder, run)
    close(feed(w, "a", toks, [70, 5, 30] + [1] * 15),
          models.expect("any-route", toks), run[2])


@pytest.mark.parametrize("run", RUNS)
class TestFarKeys:
    """Peaked scores: one key among hundreds decides."""

    def test_peaked_scores(self, models, run):
        weights = M.random_weights(M.TILED, 6)
        for k in weights:
            if k.endswith(("mix.q", "mix.k")):
                weights[k] = (weights[k].float() * 1.4).bfloat16()
        folder, cfg, _ = models("peaked", M.TILED, weights)
        toks = M.tokens(cfg, 290, 5)
        want = models.expect("peaked", toks)
        w = worker(folder, run)
        # exact runs hold their tolerance; rounding of sharp scores shows more
        limit = run[2] * (1 if run[1] == torch.float32 else 3)
        for rid, cuts in (("whole", [290]), ("pieces", [101, 2, 150, 37]),
                          ("decode", [200] + [1] * 90)):
            close(feed(w, rid, toks, cuts), want, limit, rid)
            w.finish_spans(rid)

    @pytest.mark.parametrize("change", ["first", "sink"])
    def test_faults_would_show(self, models, run, change):
        """An oracle that hides a key or the sink is far outside the
        tolerance the engine keeps."""
        folder, cfg, weights = models("tiled")
        toks = M.tokens(cfg, 60, 9)
        right = models.expect("tiled", toks)
        kept = oracle.sink_softmax

        def wrong(s, see):
            if change == "first":
                see = see.clone()
                see[1:, 0] = False
                return kept(s, see)
            return torch.softmax(s.masked_fill(~see, -1e300), -1)
        oracle.sink_softmax = wrong
        try:
            bad = oracle.forward(cfg, weights, toks)
        finally:
            oracle.sink_softmax = kept
        err = (bad - right).pow(2).mean(-1).sqrt() / right.pow(2).mean().sqrt()
        assert float(err[1:].mean()) > 2 * run[2]
        w = worker(folder, run)
        close(feed(w, "a", toks, [33] + [1] * 27), right, run[2])


@GPU
class TestRealisticSizes:
    """Head and expert sizes of a served model: the widest forms of the
    kernels, every form of the experts' products."""
    CFG = {
        "architecture": "Sezazen", "vocab": 160, "width": 512,
        "embedding": {"scale": 1.0}, "norm": {"eps": 1e-6},
        "max_positions": 1500, "loop": {"start": 1, "stop": 2, "times": 2},
        "layers": [
            M.entry(M.attention(8, 2, 128, 128, 0.11),
                    M.moe(8, 2, 320, 512)),
            M.entry(M.attention(16, 1, 192, 128, 0.09),
                    {"kind": "dense", "ff": 384}),
            M.entry(M.attention(33, 1, 64, 256, 0.15),
                    M.moe(40, 5, 64, 192)),
        ]}

    @pytest.mark.parametrize("run", RUNS[1:])
    def test_cuts_and_batches(self, models, run):
        folder, cfg, _ = models("realistic", self.CFG)
        w = worker(folder, run, blocks=160, max_model_len=1500)
        a, b = M.tokens(cfg, 450, 1), M.tokens(cfg, 200, 2)
        close(feed(w, "a", a, [300, 5, 133] + [1] * 12),
              models.expect("realistic", a), run[2])
        out = [w.forward_spans([TokenSpan("b", b[:130], list(range(130)))])]
        c = M.tokens(cfg, 700, 3)
        for i in range(70):
            spans = [TokenSpan("b", [b[130 + i]], [0])]
            if i == 3:
                spans.append(TokenSpan("c", c, list(range(700))))
            r = w.forward_spans(spans)
            out.append(r[:1])
            if i == 3:
                close(r[1:], models.expect("realistic", c), run[2], "c")
        close(torch.cat(out), models.expect("realistic", b), run[2], "b")


class TestFramework:
    def test_reader(self, models):
        folder, cfg, weights = models("odd")
        c = registry.resolve(folder)
        assert (c.vocab_size, c.hidden_size, c.num_layers) == (71, 38, 4)
        assert set(sezazen.tensor_shapes(c)) == set(weights)
        assert [(r.layer, r.cache, r.enters) for r in c.runs] == [
            (0, 0, None), (1, 1, 0), (2, 2, None), (1, 3, 1), (2, 4, None),
            (3, 5, None)]
        # every pass has pages of its own
        per = [2 * 12, 3 * 23, 8, 3 * 23, 8, 12]
        assert c.kv_bytes_per_token(2) == 2 * sum(per)
        pool = worker(folder, CPU, blocks=3).pool
        assert [p.shape[1] * p.shape[3] for p in pool.layers] == per
        assert c.layers[0].ff.shared_ff == 13
        assert c.layers[2].ff is None and c.layers[3].ff.shared_ff is None
        assert not c.has_recurrent_state
        assert c.learned_positions and c.max_position == 300

    @pytest.mark.parametrize("change,text", [
        (lambda c: c["layers"][0].update(type="other"), "unknown mixer"),
        (lambda c: c["layers"][1]["mlp"].update(kind="odd"), "unknown mlp"),
        (lambda c: c["layers"][0]["mixer"].update(kv_heads=4), "multiple"),
        (lambda c: c["layers"][0]["mlp"]["router"].update(top=6), "top 6"),
        (lambda c: c["loop"].update(stop=5), "loop"),
        (lambda c: c["loop"].update(start=3), "loop"),
        (lambda c: c["loop"].update(times=0), "loop")])
    def test_bad_configurations(self, tmp_path, change, text):
        cfg = copy.deepcopy(M.ODD)
        change(cfg)
        folder, _ = M.write_model(tmp_path, cfg, M.random_weights(M.ODD))
        with pytest.raises(ValueError, match=text):
            registry.resolve(folder)

    @pytest.mark.parametrize("name", ["pos", "loop.step", "l0.mlp.e4.down",
                                      "l0.mlp.shared.up"])
    def test_missing_tensor(self, tmp_path, name):
        w = M.random_weights(M.ODD)
        del w[name]
        folder, _ = M.write_model(tmp_path, M.ODD, w)
        with pytest.raises(ValueError, match=name):
            worker(folder, CPU, blocks=8)

    def test_positions_end_at_the_table(self, models):
        folder, cfg, _ = models("once")
        w = worker(folder, CPU, prefill_min_tokens=1)
        assert w.max_model_len == 200
        w.add_request(EngineRequest("x", [1] * 200, max_tokens=1))
        assert "context_length_exceeded" in w.step()[0].error
        toks = M.tokens(cfg, 200, 8)
        close(feed(w, "a", toks, [150, 49, 1]), models.expect("once", toks),
              CPU[2])
        with pytest.raises(ValueError, match="tokens at 200"):
            w.forward_spans([TokenSpan("a", [1], [0])])

    @pytest.mark.parametrize("run", RUNS)
    def test_prefix_cache(self, models, run):
        """Pages of another request's equal prompt serve all passes."""
        folder, cfg, weights = models("tiled")
        w = worker(folder, run, prefill_min_tokens=1)
        p = M.tokens(cfg, 70, 3)
        a = generate(w, {"a": p}, 4)["a"]
        b = generate(w, {"b": p[:64] + M.tokens(cfg, 9, 4)}, 4)["b"]
        c = generate(w, {"c": p}, 4)["c"]
        assert a.cached_tokens == 0 and b.cached_tokens == 64 \
            and c.cached_tokens == 64
        best_by_oracle(cfg, weights, p, c.all_tokens, run[2])
        best_by_oracle(cfg, weights, p[:64] + M.tokens(cfg, 9, 4),
                       b.all_tokens, run[2])

    def test_preemption_recomputes(self, models):
        folder, cfg, weights = models("odd")
        prompts = {"p": M.tokens(cfg, 40, 1), "q": M.tokens(cfg, 40, 2)}
        w = worker(folder, CPU, blocks=7, prefill_min_tokens=1)
        for r, o in generate(w, prompts, 20).items():
            best_by_oracle(cfg, weights, prompts[r], o.all_tokens, CPU[2])

    def test_temperature_samples(self, models):
        folder, cfg, _ = models("once")
        w = worker(folder, CPU, prefill_min_tokens=1)
        w.add_request(EngineRequest("t", M.tokens(cfg, 9), max_tokens=30,
                                    temperature=5.0))
        out = []
        while w.has_work:
            out += [t for o in w.step() for t in o.new_tokens]
        assert len(out) == 30 and len(set(out)) > 5

    def test_unsupported_requests_are_refused(self, models):
        folder, _, _ = models("odd")
        w = worker(folder, CPU)
        w.add_request(EngineRequest("x", [1, 2], prefill_only=True))
        out = w.step()
        assert out[0].finished and "unsupported" in out[0].error
        from llm_d_inference_scheduler_amd.node import NodeConfig, NodeRunner
        with pytest.raises(ValueError, match="hand-off"):
            NodeRunner(NodeConfig(model=registry.resolve(folder),
                                  topology="pd-combined"))

    def test_embeddings(self, models):
        folder, cfg, _ = models("odd")
        w = worker(folder, CPU, prefill_min_tokens=1)
        w.add_request(EngineRequest("e", M.tokens(cfg, 20), max_tokens=0,
                                    is_embedding=True))
        outs = []
        while w.has_work:
            outs += w.step()
        assert outs[0].kind == "embedding" and outs[0].embedding.shape == (38,)

    def test_random_init_is_seeded(self):
        from llm_d_inference_scheduler_amd.models.configs import TINY_SEZAZEN
        outs = []
        for seed in (3, 3, 4):
            w = EngineWorker(TINY_SEZAZEN, "cpu", kv_blocks=16,
                             dtype=torch.float32, seed=seed)
            outs.append(w.forward_spans([TokenSpan("a", [5, 6, 7], [2])]))
        assert torch.equal(outs[0], outs[1])
        assert not torch.equal(outs[0], outs[2])
        assert 0.01 < float(outs[0].std()) < 1e3

    def test_weight_bytes_count_everything_once(self, models):
        folder, _, weights = models("tiled")
        w = worker(folder, CPU, blocks=3)
        assert w.model.weight_bytes() >= 4 * sum(
            t.numel() for k, t in weights.items()
            if "mlp" in k or "mix" in k or k == "embed")

    @pytest.mark.parametrize("run", RUNS)
    def test_node_generates(self, models, run):
        """The node's front door: routing, scheduler, engine, completions."""
        from llm_d_inference_scheduler_amd.node import NodeConfig, NodeRunner
        from llm_d_inference_scheduler_amd.scheduling.types import LLMRequest
        folder, cfg, weights = models("tiled")
        node = NodeRunner(NodeConfig(
            model=registry.resolve(folder), device=run[0], dtype=run[1],
            kv_blocks=64, max_decode_batch=4))
        prompts = {f"n{i}": M.tokens(cfg, 20 + 9 * i, 90 + i)
                   for i in range(3)}
        for rid, p in prompts.items():
            node.submit(LLMRequest(request_id=rid, model="tiled", prompt="",
                                   prompt_tokens=list(p), max_tokens=5))
        done = {}
        for _ in range(100):
            node.step()
            for c in node.drain_completions():
                assert not c.error, c.error
                done[c.request_id] = c.tokens
            if len(done) == 3:
                break
        node.shutdown()
        assert set(done) == set(prompts)
        for rid, p in prompts.items():
            assert len(done[rid]) == 5
            best_by_oracle(cfg, weights, p, done[rid], run[2])

    def test_serve_cli_builds_from_a_folder(self, models):
        from llm_d_inference_scheduler_amd.server.__main__ import (
            build_node, parse_args)
        node = build_node(parse_args(["--model", models("odd")[0],
                                      "--device", "cpu"]))
        assert node.engine.model.cfg.hidden_size == 38
        assert node.engine.max_model_len == 300
        node.shutdown()


class TestTraceRunner:
    @pytest.mark.parametrize("device,dtype,limit", [
        ("cpu", "float32", 1e-5),
        pytest.param("cuda:0", "float32", 1e-5, marks=GPU),
        pytest.param("cuda:0", "bfloat16", 3e-2, marks=GPU)])
    def test_replay(self, models, tmp_path, monkeypatch, capsys, device,
                    dtype, limit):
        folder, cfg, _ = models("tiled")
        toks = {"x": M.tokens(cfg, 70, 30), "y": M.tokens(cfg, 50, 31),
                "z": M.tokens(cfg, 64, 32)}
        steps = [
            {"entries": [("x", 40, [0, 39])], "end": []},
            {"entries": [("x", 1, [0]), ("y", 48, [])], "end": []},
            {"entries": [("y", 1, [0]), ("x", 29, [28, 3])], "end": ["x"]},
            {"entries": [("z", 64, [63]), ("y", 1, [0])],
             "end": ["y", "z"]}]
        at, lines, want = {}, [], []
        for n, s in enumerate(steps):
            entries, rows = [], []
            for r, k, places in s["entries"]:
                lo = at.get(r, 0)
                at[r] = lo + k
                entries.append({"id": r, "tokens": toks[r][lo:lo + k],
                                "want": places})
                rows += [models.expect("tiled", toks[r])[lo + p]
                         for p in places]
            lines.append(json.dumps({"step": n, "entries": entries,
                                     "end": s["end"]}))
            want.append(rows)
        # 12 pages: z needs what x gave back
        argv = ["--model", folder, "--dtype", dtype, "--out", str(tmp_path),
                "--max-tokens", "192", "--device", device]
        text = "\n".join(lines) + "\n"
        if device == "cpu":         # the program itself
            p = subprocess.run([os.path.join(ROOT, "bin", "trace_run")] + argv,
                               input=text, capture_output=True, text=True,
                               timeout=110)
            assert p.returncode == 0, p.stderr[-2000:]
            said = p.stdout
        else:
            monkeypatch.setattr(sys, "stdin", io.StringIO(text))
            assert trace.main(argv) == 0
            said = capsys.readouterr().out
        assert [x for x in said.splitlines() if x.startswith("done")] \
            == [f"done {n}" for n in range(4)]
        for n, rows in enumerate(want):
            raw = torch.frombuffer(
                bytearray((tmp_path / f"{n}.f32").read_bytes()),
                dtype=torch.float32)
            close(raw.view(len(rows), cfg["vocab"]), torch.stack(rows),
                  limit)
