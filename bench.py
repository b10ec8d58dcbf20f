#!/usr/bin/env python3
"""Headline benchmark: decode tokens/s of the paged-attention inference path on MI355X.

    python bench.py --gpus N --steps K --warmup W
    (N>1: one rank per GPU.  Started WITHOUT torch.distributed.run, the script starts it itself as a child
    process — before anything has touched the GPU — relays the child's output and exits with its code.)

Workload: Qwen3-1.7B, bf16, kvcache_block_size=64,
hipGraph decode, max_num_seqs=256 — B=256 sequences at context 1024, synthetic token ids,
random-initialised weights at the true architecture dimensions (no checkpoints offline; throughput is
value-independent).  One "step" = one engine decode step over the whole batch: scheduler ->
input prep -> H2D -> graph replay (28 layers + LM head + sampler) -> D2H of the B tokens ->
postprocess.  value = B * K / wall time (max over ranks).  With N>1 the same model runs
tensor-parallel over N GPUs (RCCL all-reduce over xGMI): total work fixed => "strong" scaling.

What else `--gpus N` puts on the line (BASELINE.json's metric is "Qwen3-1.7B TP=1 & Qwen2-7B TP=1/2/4/8", config 5 is
Qwen2-72B TP=8): see ``record_plan`` -- N=1: sampled decode + prefill for the headline model, Qwen2-7B decode + prefill;
N=2/4: Qwen2-7B decode + prefill at TP=N; N=8: the Qwen2-7B TP=8 rejection (28/4 heads, as in the reference) and
Qwen2-72B TP=8 decode with its per-GPU KV pool.  No scaling curve has been measured on hardware by the builder (one-GPU
boxes): the N>1 path is rehearsed with ranks time-slicing one card (profiles/r04_bench_lines.md).

Also reported on the same line:
  roofline     — the dominant kernel (paged-KV decode attention): algorithmic bytes per launch /
                 average launch time, timed with HIP events on the launching stream on the LIVE
                 block tables / context lengths / KV cache of this run
  projection_roofline — the decode-batch projection kernel (linear_mid_m_kernel): weight bytes / HIP-event time of the four
                 projections of every layer replayed from a captured graph (HBM bound), next to the bound that binds it at
                 256 rows: what one CU must take in, (BM + BN) x K x 2 bytes per workgroup, at the guide's 66-73 GB/s per CU
  step_roofline — the whole decode step: weights touched once + the KV bytes of the batch, per GPU, over ms_per_step
  cpu_baseline — the CPU restatement of the reference's eager path (oracle/, "port") timed on this
                 host's cores on a bounded sample of the same model (one untimed warm-up step, then the
                 median of a fixed number of steps), plus BASELINE config 1 (OPT-125M fp32, the preset of
                 the reference's examples/cpu_inference_opt.py) as `config1`
  secondary    — the rest of BASELINE.json's metric under the same clock (``record_plan``); every prefill record carries
                 a roofline object of the flash kernel (HIP-event time of the mv_prefill_varlen launches of one extra
                 eager batch, flops = sum 4 H D (Sq Sk - Sq (Sq - 1) / 2), peak 2.5 PFLOP/s dense bf16, MFMA-busy quoted
                 from the committed PMC profile)
  allreduce_probe — (N>1) HIP-event time of the tensor-parallel all-reduce launches of eager probe steps, per rank
"""
from __future__ import annotations

import argparse
import json
import os
import statistics
import subprocess
import sys
import tempfile
import time

ROOT = os.path.dirname(os.path.abspath(__file__))
sys.path.insert(0, ROOT)

import torch  # noqa: E402

MODELS = {
    # public HF config.json values
    "qwen3-1.7b": dict(model_type="qwen3", architectures=["Qwen3ForCausalLM"], hidden_size=2048,
                       num_hidden_layers=28, num_attention_heads=16, num_key_value_heads=8, head_dim=128,
                       intermediate_size=6144, vocab_size=151936, max_position_embeddings=40960,
                       rms_norm_eps=1e-6, rope_theta=1000000.0, tie_word_embeddings=True, hidden_act="silu",
                       attention_bias=False, torch_dtype="bfloat16", eos_token_id=151645),
    "qwen3-0.6b": dict(model_type="qwen3", architectures=["Qwen3ForCausalLM"], hidden_size=1024,
                       num_hidden_layers=28, num_attention_heads=16, num_key_value_heads=8, head_dim=128,
                       intermediate_size=3072, vocab_size=151936, max_position_embeddings=40960,
                       rms_norm_eps=1e-6, rope_theta=1000000.0, tie_word_embeddings=True, hidden_act="silu",
                       attention_bias=False, torch_dtype="bfloat16", eos_token_id=151645),
    "qwen2-7b": dict(model_type="qwen2", architectures=["Qwen2ForCausalLM"], hidden_size=3584,
                     num_hidden_layers=28, num_attention_heads=28, num_key_value_heads=4,
                     intermediate_size=18944, vocab_size=152064, max_position_embeddings=32768,
                     rms_norm_eps=1e-6, rope_theta=1000000.0, tie_word_embeddings=False, hidden_act="silu",
                     torch_dtype="bfloat16", eos_token_id=151645),
    "qwen2-72b": dict(model_type="qwen2", architectures=["Qwen2ForCausalLM"], hidden_size=8192,
                      num_hidden_layers=80, num_attention_heads=64, num_key_value_heads=8,
                      intermediate_size=29568, vocab_size=152064, max_position_embeddings=32768,
                      rms_norm_eps=1e-6, rope_theta=1000000.0, tie_word_embeddings=False, hidden_act="silu",
                      torch_dtype="bfloat16", eos_token_id=151645),
}


def _mofarax(like: str, side_dim: int = 128, layers: int = 20, loop=(8, 12, 3), chunk: int = 2048) -> dict:
    """A Mofarax configuration whose layer runs (28: 20 layers, four of them passed three times) have the sizes of
    ``like``'s layers; the keys behind the first line are what this script itself asks of a model."""
    c = MODELS[like]
    heads, kv, width, vocab = (c[k] for k in ("num_attention_heads", "num_key_value_heads", "hidden_size", "vocab_size"))
    dim = c.get("head_dim") or width // heads
    mixer = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "mask": {"size": chunk},
             "rot": {"base": c["rope_theta"], "dims": dim}}
    layer = {"type": "attention", "mixer": mixer, "mlp": {"kind": "dense", "ff": c["intermediate_size"]}}
    assert layers + (loop[1] - loop[0]) * (loop[2] - 1) == c["num_hidden_layers"]
    return dict(architecture="Mofarax", vocab=vocab, width=width, embedding={"scale": width ** 0.5}, norm={"eps": 1e-6},
                layers=[layer] * layers, loop=dict(zip(("start", "stop", "times"), loop)), token_side={"dim": side_dim},
                like=like, chunk=chunk, vocab_size=vocab, hidden_size=width, num_attention_heads=heads, num_key_value_heads=kv,
                head_dim=dim, intermediate_size=c["intermediate_size"])


def _kugulorn(like: str, q_rank: int, ssm_heads: int, groups: int, pairs: int, window: int = 2048, kv_rank: int = 512, rot: int = 64,
              state: int = 128) -> dict:
    """A Kugulorn configuration of ``pairs`` x [state space layer, latent attention layer with a feed-forward] with ``like``'s
    width, heads and feed-forward; as many pairs as make the layers' weights ``like``'s.  Every second attention layer reads the
    latents of the one before."""
    c = MODELS[like]
    heads, width, vocab = c["num_attention_heads"], c["hidden_size"], c["vocab_size"]
    ssm = {"type": "mamba2", "mlp": None, "mixer": {"heads": ssm_heads, "vdim": 64, "state": state, "groups": groups, "conv": 4,
                                                   "norm_groups": groups}}
    layers = []
    for i in range(pairs):
        mixer = {"heads": heads, "dim": 128, "rot_dim": rot, "vdim": 128, "q_rank": q_rank, "kv_rank": kv_rank,
                 "mask": {"size": window}, "rot": {"base": c["rope_theta"], "dims": rot}, "scale": (128 + rot) ** -0.5}
        if i % 2:
            mixer["kv_from"] = len(layers) - 1
        layers += [ssm, {"type": "latent_attention", "mixer": mixer,
                         "mlp": {"kind": "dense", "ff": c["intermediate_size"], "limit": 7.0}}]
    return dict(architecture="Kugulorn", vocab=vocab, width=width, norm={"eps": 1e-6}, residual_mult=0.5, layers=layers, like=like,
                window=window, vocab_size=vocab, hidden_size=width, num_attention_heads=heads, num_key_value_heads=1,
                head_dim=kv_rank + rot, intermediate_size=c["intermediate_size"])


def _pununex(like: str, peer: str, pairs: int, window: int = 2048, experts: int = 32, rank: int = 128) -> dict:
    """A Pununex configuration of ``pairs`` x [gated delta rule with a dense feed-forward, attention beside a gated delta rule with
    experts], with ``like``'s width, heads and feed-forward: a token's experts (4, and a shared one) have its size together.  As many
    pairs as make the weights that a token uses ``like``'s; ``peer``: the model it is compared with."""
    c = MODELS[like]
    heads, kv, width, ff = (c[k] for k in ("num_attention_heads", "num_key_value_heads", "hidden_size", "intermediate_size"))
    delta = {"heads": heads, "kv_heads": heads // 2, "dim": 128, "vdim": 128, "conv": 4}
    left = {"heads": heads, "kv_heads": kv, "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "softcap": 50.0,
            "mask": {"size": window, "keep_first": 8}}
    right = {"heads": heads // 2, "kv_heads": heads // 2, "dim": 128, "vdim": 128, "conv": 4, "rank": rank}
    moe = {"kind": "moe", "router": {"experts": experts, "identity": 2, "top": 4, "scale": 2.5,
                                     "groups": {"count": 2, "keep": 1}}, "expert": {"ff": ff // 8}, "shared": {"ff": ff // 2}}
    layers = [{"type": "delta", "mixer": delta, "mlp": {"kind": "dense", "ff": ff}},
              {"type": "parallel", "mixer": {"left": left, "right": right, "left_scale": 0.7, "right_scale": 0.7}, "mlp": moe}] * pairs
    return dict(architecture="Pununex", vocab=c["vocab_size"], width=width, norm={"eps": 1e-6}, layers=layers, like=peer, window=window,
                embedding={"bigram": {"buckets": 65521, "mul_prev": 131, "mul_cur": 71}}, vocab_size=c["vocab_size"], hidden_size=width,
                num_attention_heads=heads, num_key_value_heads=kv, head_dim=128, intermediate_size=ff)


def _semezen(like: str, peer: str, pairs: int, window: int = 2048, experts: int = 32, streams: int = 4) -> dict:
    """A Semezen configuration of ``pairs`` x [attention with a dense feed-forward, gated running mean with experts], with ``like``'s
    width, heads and feed-forward weights (two matrices have the size of three, a token's 8 experts together too); as many pairs as
    make the weights that a token uses ``like``'s.  ``peer``: the model it is compared with."""
    c = MODELS[like]
    heads, kv, width, ff = (c[k] for k in ("num_attention_heads", "num_key_value_heads", "hidden_size", "intermediate_size"))
    mixer = {"heads": heads, "kv_heads": kv, "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "mask": {"size": window},
             "rot": {"base": c["rope_theta"], "dims": 64, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}}
    moe = {"kind": "moe", "router": {"experts": experts, "top": 8}, "expert": {"ff": ff // 8, "limit": 7.0}}
    layers = [{"type": "attention", "mixer": mixer, "mlp": {"kind": "dense", "ff": ff * 3 // 2}},
              {"type": "mingru", "mixer": {"width": heads * 128}, "mlp": moe}] * pairs
    return dict(architecture="Semezen", vocab=c["vocab_size"], width=width, streams=streams, norm={"eps": 1e-6}, layers=layers, like=peer,
                window=window, vocab_size=c["vocab_size"], hidden_size=width, num_attention_heads=heads, num_key_value_heads=kv,
                head_dim=128, intermediate_size=ff)


DESIGNS = {"mofarax": {"mofarax-0.6b": "qwen3-0.6b", "mofarax-1.7b": "qwen3-1.7b", "mofarax-7b": "qwen2-7b"},
           "kugulorn": {"kugulorn-0.6b": "qwen3-0.6b", "kugulorn-1.7b": "qwen3-1.7b", "kugulorn-7b": "qwen2-7b"},
           # (beside the design that also mixes attention with a recurrence)
           "pununex": {"pununex-0.6b": "kugulorn-0.6b", "pununex-1.7b": "kugulorn-1.7b", "pununex-7b": "kugulorn-7b"},
           # (beside the design with windowed attention, a recurrence and experts too)
           "semezen": {"semezen-0.6b": "pununex-0.6b", "semezen-1.7b": "pununex-1.7b", "semezen-7b": "pununex-7b"}}
MODELS.update({name: _mofarax(like) for name, like in DESIGNS["mofarax"].items()})
MODELS.update({"kugulorn-0.6b": _kugulorn("qwen3-0.6b", 512, 32, 1, 19), "kugulorn-1.7b": _kugulorn("qwen3-1.7b", 768, 64, 1, 19),
               "kugulorn-7b": _kugulorn("qwen2-7b", 1536, 112, 2, 21)})
MODELS.update({f"pununex-{s}": _pununex(like, f"kugulorn-{s}", n) for s, like, n in
               (("0.6b", "qwen3-0.6b", 12), ("1.7b", "qwen3-1.7b", 13), ("7b", "qwen2-7b", 13))})
MODELS.update({f"semezen-{s}": _semezen(like, f"pununex-{s}", 13) for s, like in
               (("0.6b", "qwen3-0.6b"), ("1.7b", "qwen3-1.7b"), ("7b", "qwen2-7b"))})
DESIGN_DECODE = ((256, 1024), (16, 1024), (1, 1024))      # (batch, context) of a design's decode records
DESIGN_PREFILL = ((16, 1024), (4, 4096))
HBM_PEAK_GBS = 8000.0  # MI355X_MICROARCH.md: HBM3E 8.0 TB/s spec (6.29 TB/s measured copy ceiling)
MFMA_PEAK_TFLOPS = 2500.0  # MI355X_MICROARCH.md: ~2.5 PFLOP/s dense bf16 (the 5 PF headline includes 2:1 sparsity)
L2_INGEST_GBS_PER_CU = (66.0, 73.0)  # MI355X_MICROARCH.md "Indexed rows: gather into LDS": rows shared by every workgroup, served by the XCD's L2
PREFILL_CASES = ((16, 1024), (4, 4096), (64, 256))        # config 4 prompt shapes
SAMPLED = dict(temperature=0.6, top_p=0.95, top_k=40)      # reference examples/cpu_inference_opt.py:153-158
_T0 = time.perf_counter()


def note(msg: str) -> None:
    """Progress on stderr (the JSON line on stdout stays the only stdout output): a long multi-record run must not look hung."""
    if int(os.environ.get("RANK", "0")) == 0:
        print(f"[bench +{time.perf_counter() - _T0:6.1f}s] {msg}", file=sys.stderr, flush=True)


def parse(argv=None):
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=64)
    ap.add_argument("--warmup", type=int, default=8)
    ap.add_argument("--model", default="qwen3-1.7b", choices=list(MODELS))
    ap.add_argument("--batch", type=int, default=256)
    ap.add_argument("--ctx", type=int, default=1024)
    ap.add_argument("--eager", action="store_true", help="enforce_eager (no hipGraph)")
    ap.add_argument("--synthetic-kv", action="store_true",
                    help="fill the KV cache with random values instead of running the prompt prefill")
    ap.add_argument("--auto-kv", action="store_true",
                    help="size the KV pool from free HBM (num_kvcache_blocks=-1: the DEFAULT user path, LLM(Config()); "
                         "1.5 %% slower than the explicit pool on the headline, profiles/r03_kv_stride_probe.md) instead of "
                         "allocating exactly what this workload needs")
    ap.add_argument("--no-cpu-baseline", action="store_true")
    ap.add_argument("--no-secondary", action="store_true",
                    help="skip the secondary records (the rest of BASELINE.json's metric: record_plan)")
    ap.add_argument("--cpu-steps", type=int, default=5, help="timed CPU-baseline steps (median), after one warm-up")
    ap.add_argument("--rehearse-n8", action="store_true",
                    help="(with --gpus 2, ranks sharing one card) run the N = 8 record flow on stand-ins: a Qwen2-7B-like model "
                         "whose heads do not divide by 2 (-> the rejection record) and a 4-layer model at Qwen2-72B's per-layer "
                         "dimensions on an explicit KV pool; the records are marked as a rehearsal")
    ap.add_argument("--design", choices=list(DESIGNS),
                    help="instead of the headline: decode and prefill throughput of this model design at several sizes, each "
                         "beside the closest other model with layers of the same size (one GPU, random weights)")
    ap.add_argument("--cpu-config1-only", action="store_true",
                    help="run only the CPU leg of BASELINE config 1 (OPT-125M fp32, reference preset) and print it")
    return ap.parse_args(argv)


def launch_command(args, script=None, port=None):
    """The child a bare ``python bench.py --gpus N`` (N > 1) starts: torch.distributed.run, one rank per GPU, the
    same arguments.  Separate from main() so that a host test can check it."""
    if port is None:
        import socket

        with socket.socket(socket.AF_INET, socket.SOCK_STREAM) as sock:
            sock.bind(("127.0.0.1", 0))
            port = sock.getsockname()[1]
    cmd = [sys.executable, "-m", "torch.distributed.run", "--nnodes=1", f"--nproc-per-node={args.gpus}",
           "--master-addr", "127.0.0.1", "--master-port", str(port), script or os.path.abspath(__file__),
           "--gpus", str(args.gpus), "--steps", str(args.steps), "--warmup", str(args.warmup),
           "--model", args.model, "--batch", str(args.batch), "--ctx", str(args.ctx)]
    for flag in ("eager", "synthetic_kv", "auto_kv", "no_cpu_baseline", "no_secondary", "rehearse_n8"):
        if getattr(args, flag):
            cmd.append("--" + flag.replace("_", "-"))
    return cmd


def tp_allowed(model: str, tp: int) -> bool:
    """The reference's divisibility rule (models/qwen_base.py:95-104): q heads and kv heads must divide by the TP degree."""
    c = MODELS[model]
    return c["num_attention_heads"] % tp == 0 and c["num_key_value_heads"] % tp == 0 and c["vocab_size"] % tp == 0


def record_plan(gpus: int, model: str = "qwen3-1.7b", batch: int = 256, ctx: int = 1024) -> list[dict]:
    """What one ``bench.py --gpus N`` run measures, in order (the first entry is the driver's headline, the others become
    ``secondary``).  metric = "decode tokens/sec/GPU + prefill tok/s, Qwen3-1.7B TP=1 & Qwen2-7B
    TP=1/2/4/8"; config 5 = Qwen2-72B TP=8, max_model_len=4096, 288 GB KV sizing.

      N=1    headline model: greedy decode (headline), sampled decode (the reference's preset), prefill on the three config-4
             shapes; Qwen2-7B: greedy decode, prefill on the three shapes
      N=2,4  headline model at TP=N (strong scaling point); Qwen2-7B at TP=N: greedy decode, prefill 16x1024 / 4x4096
      N=8    headline model at TP=8; Qwen2-7B TP=8 -> "rejected, as in reference" (28/4 heads); Qwen2-72B at TP=8
             (config 5): greedy decode B=256 ctx=1024 on a KV pool sized from free HBM, max_model_len=4096
    Pure host logic (tests/test_bench_host.py)."""
    plan = [dict(kind="decode", model=model, tp=gpus, batch=batch, ctx=ctx, sampling="greedy", headline=True)]
    if gpus == 1:
        plan.append(dict(kind="decode", model=model, tp=1, batch=batch, ctx=ctx, sampling="sampled"))
        plan += [dict(kind="prefill", model=model, tp=1, prompts=n, prompt_len=ln) for n, ln in PREFILL_CASES]
        if model != "qwen2-7b":
            plan.append(dict(kind="decode", model="qwen2-7b", tp=1, batch=256, ctx=1024, sampling="greedy"))
            plan += [dict(kind="prefill", model="qwen2-7b", tp=1, prompts=n, prompt_len=ln) for n, ln in PREFILL_CASES]
        return plan
    if tp_allowed("qwen2-7b", gpus):
        if model != "qwen2-7b":
            plan.append(dict(kind="decode", model="qwen2-7b", tp=gpus, batch=256, ctx=1024, sampling="greedy"))
        plan += [dict(kind="prefill", model="qwen2-7b", tp=gpus, prompts=n, prompt_len=ln) for n, ln in PREFILL_CASES[:2]]
    else:
        plan.append(dict(kind="rejected", model="qwen2-7b", tp=gpus))
    if gpus == 8:
        plan.append(dict(kind="decode", model="qwen2-72b", tp=8, batch=256, ctx=1024, sampling="greedy", auto_kv=True,
                         max_model_len=4096))
    return plan


def build_engine(args, workdir, model=None, max_model_len=None, auto_kv=None):
    from minivllm_amd import LLM, Config

    model = model or args.model
    os.makedirs(workdir, exist_ok=True)
    with open(os.path.join(workdir, "config.json"), "w") as f:
        json.dump(MODELS[model], f)
    max_len = max_model_len or max(4096, args.ctx + args.steps + args.warmup + 64)
    auto_kv = args.auto_kv if auto_kv is None else auto_kv
    cfg = Config(workdir, dtype="bfloat16", kvcache_block_size=64, max_num_seqs=args.batch,
                 max_model_len=max_len, max_num_batched_tokens=max(16384, max_len),
                 tensor_parallel_size=args.gpus, enforce_eager=args.eager, load_format="dummy", seed=0,
                 num_kvcache_blocks=-1 if auto_kv else
                 args.batch * (-(-(args.ctx + args.steps + args.warmup + 8) // 64) + 1))
    return LLM(cfg)


def fill_prompts(engine, args, model=None, sampling=None, seed=0):
    """B requests of ctx synthetic tokens each -> running sequences with allocated blocks."""
    from minivllm_amd import SamplingParams

    g = torch.Generator().manual_seed(seed)
    vocab = MODELS[model or args.model]["vocab_size"]
    sp = SamplingParams(max_tokens=args.steps + args.warmup + 16, ignore_eos=True, **(sampling or dict(temperature=0.0)))
    for _ in range(args.batch):
        engine.add_request(torch.randint(0, vocab, (args.ctx,), generator=g).tolist(), sp)
    prefill_tokens, t0 = 0, time.perf_counter()
    if args.synthetic_kv:
        ex = engine.model_runner.inference_executor
        ex.kv_cache.normal_(0.0, 1.0)
        while engine.scheduler.waiting:
            batch, is_prefill = engine.scheduler.schedule()
            assert is_prefill
            engine.scheduler.postprocess(batch, [1] * len(batch))
        return None
    while engine.scheduler.waiting:
        _, n = engine.step()
        prefill_tokens += max(n, 0)
    torch.cuda.synchronize()
    return prefill_tokens / (time.perf_counter() - t0)


class _EventProbe:
    """Brackets calls with HIP event pairs recorded on the stream the call launches on (torch's current stream)."""

    def __init__(self):
        self.pairs: dict[str, list] = {}

    def wrap(self, name, real, keep=lambda out: True):
        def timed(*a, **kw):
            stream = torch.cuda.current_stream()
            e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
            e0.record(stream)
            out = real(*a, **kw)
            e1.record(stream)
            if keep(out):
                self.pairs.setdefault(name, []).append((e0, e1))
            return out
        return timed

    def times_us(self, name):
        return [a.elapsed_time(b) * 1e3 for a, b in self.pairs.get(name, [])]


def _event_pair_floor_us(device) -> float:
    """What an event pair itself costs: the same bracket around a one-element fill, inside a stream that is busy."""
    tiny, floor = torch.zeros(1, device=device), []
    busy = torch.empty(256 << 20, dtype=torch.uint8, device=device)
    for _ in range(20):
        busy.zero_()                        # ~50 us of work ahead of the pair: the host is not what it times
        e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
        e0.record()
        tiny.zero_()
        e1.record()
        floor.append((e0, e1))
    torch.cuda.synchronize()
    del busy
    return sorted(a.elapsed_time(b) for a, b in floor)[len(floor) // 2] * 1e3


def decode_roofline(engine, args, model=None):
    """Average duration of the paged-decode launches of REAL decode steps of this run, measured with
    HIP events on the launching stream: the executor is switched to eager for a few extra steps and
    every mv_paged_decode launch (one per layer, in situ between the GEMMs, on the live block
    tables / context lengths / KV cache) is bracketed by an event pair; the host runs ahead of the GPU (see below).
    With N > 1 the same probe steps also bracket every tensor-parallel all-reduce launch (-> allreduce_probe)."""
    import torch.distributed as dist

    from minivllm_amd import hip_ops, parallel_state
    from minivllm_amd.layers import attention as attn_mod

    model = model or args.model
    ex = engine.model_runner.inference_executor
    seqs = list(engine.scheduler.running)
    lens = [len(s) for s in seqs]
    L, nb, bs, hkv, d = ex.kv_cache.shape[1:]
    heads = MODELS[model]["num_attention_heads"] // args.gpus
    probe = _EventProbe()
    # the launch is mv_paged_decode, or mv_rope_paged_decode where the layer folds RoPE + the K/V store into it
    reals = {"paged_decode": hip_ops.paged_decode, "rope_paged_decode": hip_ops.rope_paged_decode}
    ar = parallel_state.get_custom_all_reduce() if args.gpus > 1 else None
    ar_reals = {}
    if ar is not None:
        ar_reals = {"all_reduce": ar.all_reduce, "all_reduce_add_rmsnorm": ar.all_reduce_add_rmsnorm}
    real_dist_ar = dist.all_reduce
    was_eager = ex.enforce_eager
    ex.enforce_eager = True
    # (steps of <= 16 rows run all layers in one persistent launch: the probe times the attention kernel on its own, so
    #  its steps take the multi-launch path, which computes the same bits)
    from minivllm_amd.glue import qwen as _qwen
    was_persistent, _qwen.PERSISTENT = _qwen.PERSISTENT, False
    # (Events cannot be recorded inside a captured graph on ROCm — "External events are disallowed in rocm",
    # tools/dbg/ext_event_probe.py — so the probe steps are eager.  Keeping the host ahead of the GPU with a spin
    # kernel in front of each probe step changes nothing (180 vs 178 us): what an event pair adds to the ~168 us
    # rocprofv3 sees for this kernel inside the graph is the two event packets themselves, reported below as
    # `event_pair_floor_us` = the same pair around a one-element fill.)
    probe_steps = 3
    try:
        engine.step()                       # eager warm-up step (kernels already resident)
        for name, real in reals.items():
            # (None: the fused form declined the layout, the plain launch follows)
            setattr(attn_mod.hip_ops, name, probe.wrap("decode", real, keep=lambda out: out is not None))
        for name, real in ar_reals.items():
            setattr(ar, name, probe.wrap("p2p_" + name, real))
        if args.gpus > 1:
            dist.all_reduce = probe.wrap("backend_all_reduce", real_dist_ar)
        for _ in range(probe_steps):
            engine.step()
    finally:
        for name, real in reals.items():
            setattr(attn_mod.hip_ops, name, real)
        for name in ar_reals:
            delattr(ar, name)               # the instance attribute shadowed the method
        dist.all_reduce = real_dist_ar
        ex.enforce_eager = was_eager
        _qwen.PERSISTENT = was_persistent
    torch.cuda.synchronize()
    times = [t * 1e-3 for t in probe.times_us("decode")]      # ms
    assert len(times) == probe_steps * L
    floor_us = _event_pair_floor_us(ex.device)
    # an event pair also spans whatever the HOST does between recording the first event and enqueuing the
    # kernel while the GPU is idle (eager probe steps are launch-bound): a rare host stall there (seen: one
    # ~170 ms gap in 84 launches) is not kernel time.  Launches above 3x the median are left out and counted.
    med = sorted(times)[len(times) // 2]
    kept = [t for t in times if t <= 3 * med]
    sec = sum(kept) * 1e-3 / len(kept)
    esz = ex.dtype.itemsize
    lens = [n + 1 + probe_steps // 2 for n in lens]   # context length at the middle probe step
    algo = sum(lens) * 2 * hkv * d * esz + 2 * len(seqs) * heads * d * esz + sum(-(-n // bs) for n in lens) * 4
    gbs = algo / sec / 1e9
    # HBM traffic from the PMC counters (separate rocprofv3 --pmc passes, corrected as the microarch guide
    # prescribes): measured on the same kernel / head layout at B=256, ctx=1024 and scaled by bytes
    traffic = src = None
    for pmc in ("r04_pmc_decode.json", "r03_pmc_decode.json", "r02_pmc_decode.json"):
        path = os.path.join(ROOT, "profiles", pmc)
        if os.path.exists(path) and args.gpus == 1 and traffic is None:
            with open(path) as f:
                for name, rec in json.load(f)["kernels"].items():
                    if model in name:
                        traffic, src = int(algo * rec["ratio"]), pmc
    cfgm = MODELS[model]
    kernel = ("paged_decode_mfma_kernel" if cfgm["num_attention_heads"] // cfgm["num_key_value_heads"] >= 4
              else "paged_decode_kernel")
    roof = {"bound": "hbm", "kernel": kernel, "achieved": round(gbs, 1), "peak": HBM_PEAK_GBS,
            "unit": "GB/s", "frac": round(gbs / HBM_PEAK_GBS, 4), "traffic": traffic,
            "traffic_source": f"profiles/{src} (rocprofv3 --pmc FETCH_SIZE x2 + WRITE_SIZE in separate passes on this kernel and head layout at B=256 ctx=1024, per launch, scaled to this run's context; counters cannot be read inside a timed run)" if traffic else None,
            "heads_per_rank": [heads, hkv],
            "bytes_per_launch": algo, "us_per_launch": round(sec * 1e6, 2), "event_pair_floor_us": round(floor_us, 2),
            "launches_timed": len(kept),
            "launches_discarded_host_stall": len(times) - len(kept)}
    ar_probe = None
    if args.gpus > 1:
        ar_probe = {"probe_steps": probe_steps, "event_pair_floor_us": round(floor_us, 2)}
        for name in ("p2p_all_reduce", "p2p_all_reduce_add_rmsnorm", "backend_all_reduce"):
            t = probe.times_us(name)
            if t:
                m = statistics.median(t)
                keep = [v for v in t if v <= 3 * m]
                ar_probe[name] = {"launches_per_step": round(len(t) / probe_steps, 1), "median_us": round(m, 2),
                                  "us_per_step": round(sum(keep) / len(keep) * len(t) / probe_steps, 1)}
    return roof, ar_probe


@torch.inference_mode()
def _graph_time_us(fn, launches: int, reps: int = 5) -> float:
    """Microseconds per launch of ``fn`` (which enqueues ``launches`` kernels on the current stream): captured into a
    hipGraph -- how the decode step itself runs them -- and replayed between one HIP event pair per replay (on the
    replaying stream), median over ``reps``; the event pair and the replay's fixed cost are spread over all launches."""
    side = torch.cuda.Stream()
    side.wait_stream(torch.cuda.current_stream())
    with torch.cuda.stream(side):
        fn()
    torch.cuda.current_stream().wait_stream(side)
    graph = torch.cuda.CUDAGraph()
    with torch.cuda.graph(graph):
        fn()
    graph.replay()
    torch.cuda.synchronize()
    pairs = []
    for _ in range(reps):
        e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
        e0.record()
        graph.replay()
        e1.record()
        pairs.append((e0, e1))
    torch.cuda.synchronize()
    del graph
    return statistics.median(a.elapsed_time(b) for a, b in pairs) * 1e3 / launches


def projection_plan(kind: str, rows: int, n: int, k: int) -> dict | None:
    """Tile, K split, workgroup count and per-CU ingest of the mv_linear_mid_m launch that ``layers/linear.py`` picks for
    this projection (None: the library GEMM).  ``n`` = output features (gated: the intermediate size).  The ingest
    figure is what the busiest CU must take in: every workgroup reads its BM rows of x and its BN weight rows over its
    K slice, (BM + BN) x K/splits x 2 bytes, and a CU runs ceil(workgroups / 256) of them.  Host logic."""
    from minivllm_amd.layers.linear import MID_CFGS, mid_plan

    cfg, splits = mid_plan(kind, rows, n, k)
    if not cfg:
        return None
    bm, bn, _ = MID_CFGS[cfg]
    bno = bn // 2 if kind == "gated" else bn
    wgs = -(-rows // bm) * -(-n // bno) * splits
    per_cu = -(-wgs // 256) * (bm + bn) * (k // splits) * 2
    lo, hi = L2_INGEST_GBS_PER_CU
    return {"cfg": cfg, "tile": [bm, bn], "k_splits": splits, "workgroups": wgs, "ingest_bytes_per_cu": per_cu,
            "ingest_bound_us": [round(per_cu / hi / 1e3, 2), round(per_cu / lo / 1e3, 2)]}


def projection_roofline(engine, rows: int):
    """The decode-batch projection kernel (csrc/linear_mid_m.hip) on this engine's own weights at ``rows`` tokens: per
    projection kind, one launch per LAYER (28 different weight matrices, so every launch streams its weights from HBM
    like the step does) captured into a graph and replayed; weight bytes / time against the HBM peak, and next to it the
    per-CU ingest bound (``projection_plan``) -- at 256 rows the kernel is bound by how fast a CU takes bytes in, not
    by HBM (profiles/r03_mid_m_ablation.md), and 0.2 of 8 TB/s says little without that second number."""
    from minivllm_amd import hip_ops
    from minivllm_amd.layers.linear import linear, mid_m

    ex = engine.model_runner.inference_executor
    if not hasattr(ex.model, "model"):
        return None               # (a model without separate q/k/v, o, gate/up and down projections)
    layers = list(ex.model.model.layers)
    dev, dt = ex.device, ex.dtype
    g = torch.Generator(device=dev).manual_seed(7)
    kinds = (("qkv_proj", lambda l: l.self_attn.qkv_proj, "col"), ("o_proj", lambda l: l.self_attn.o_proj, "row"),
             ("gate_up_proj", lambda l: l.mlp.gate_up_proj, "gated"), ("down_proj", lambda l: l.mlp.down_proj, "row"))
    per, tot_b, tot_us, tot_lo, tot_hi = [], 0, 0.0, 0.0, 0.0
    for name, get, kind in kinds:
        mods = [get(l) for l in layers]
        w = mods[0].weight
        n, k = (w.shape[0] // 2 if kind == "gated" else w.shape[0]), w.shape[1]
        x = torch.randn((rows, k), device=dev, dtype=torch.float32, generator=g).mul_(0.05).to(dt)
        # the kind layers/linear.py resolves: a row-parallel projection may K-split into fp32 partials only on a single
        # rank (RowParallelLinear.forward), and a bias forces the plain form (linear())
        if kind == "row":
            eff = "row" if mods[0].tp_size == 1 and mods[0].bias is None else "col"
        else:
            eff = kind
        ours = mid_m(x, mods[0].weight_packed) and hip_ops.linear_mid_m_ok(x, n)
        plan = projection_plan(eff, rows, n, k) if ours else None
        if kind == "gated":
            if plan is None:
                continue          # (library GEMM + SiluAndMul launch: not this kernel)

            def run(mods=mods, x=x, n=n, cfg=plan["cfg"]):
                for m in mods:
                    hip_ops.gate_up_silu_mid_m(x, m.weight_packed, n, cfg)
        else:
            def run(mods=mods, x=x, eff=eff, row=kind == "row"):
                for m in mods:
                    linear(x, m.weight, None if row and m.tp_rank != 0 else m.bias, m.weight_packed, eff)
        us = _graph_time_us(run, len(mods))
        wbytes = w.numel() * w.element_size()
        rec = {"projection": name, "out_features": n, "in_features": k, "weight_bytes": wbytes, "us_per_launch": round(us, 2),
               "GBs": round(wbytes / us / 1e3, 1), "frac_of_hbm_peak": round(wbytes / us / 1e3 / HBM_PEAK_GBS, 4),
               "kernel": "linear_mid_m_kernel" if plan else "library GEMM (hipBLASLt)"}
        if plan:
            rec.update(plan)
            rec["frac_of_ingest_bound"] = [round(b / us, 3) for b in plan["ingest_bound_us"]]
            tot_lo += plan["ingest_bound_us"][0]
            tot_hi += plan["ingest_bound_us"][1]
        per.append(rec)
        tot_b += wbytes
        tot_us += us
    if not per:
        return None
    gbs = tot_b / tot_us / 1e3
    all_ours = all("cfg" in r for r in per)
    return {"bound": "hbm", "kernel": "linear_mid_m_kernel", "rows": rows,
            "achieved": round(gbs, 1), "peak": HBM_PEAK_GBS, "unit": "GB/s", "frac": round(gbs / HBM_PEAK_GBS, 4),
            "weight_bytes_per_layer": tot_b, "us_per_layer": round(tot_us, 2), "launches_per_layer": len(per),
            "second_bound": None if not all_ours else {
                "what": "per-CU L2 ingest: every workgroup takes in (BM + BN) x K/splits x 2 bytes (its rows of x from L2, its weight "
                        "rows), the busiest CU ceil(workgroups / 256) of them, at the guide's 66-73 GB/s per CU for rows served by the "
                        "XCD's L2 (MI355X_MICROARCH.md, 'Indexed rows: gather into LDS'); launch fill / drain not included",
                "GBs_per_cu": list(L2_INGEST_GBS_PER_CU), "bound_us_per_layer": [round(tot_lo, 2), round(tot_hi, 2)],
                "frac": [round(tot_lo / tot_us, 3), round(tot_hi / tot_us, 3)]},
            "timing": f"one launch per layer ({len(layers)} weight matrices) captured into a hipGraph, replayed between one HIP event pair "
                      "on the replaying stream, median of 5 replays / launches",
            "per_projection": per}


def step_roofline(engine, model, batch, ctx_mid, ms_per_step):
    """The whole decode step against HBM: per GPU, every matrix weight of this rank touched once (embedding
    rows excluded, the tied / untied LM head shard included) + the K/V bytes of the batch at its mean context."""
    ex = engine.model_runner.inference_executor
    seen, wbytes = set(), 0
    # weights of looped layers are read once a pass
    passes = {id(m): len(layer.attn) for layer in getattr(ex.model, "stack", []) if hasattr(layer, "attn") for m in layer.modules()}
    for mod in ex.model.modules():
        w = getattr(mod, "weight", None)
        if w is None or w.dim() != 2 or w.data_ptr() in seen:
            continue
        if hasattr(mod, "input_size") or type(mod).__name__ == "ParallelLMHead":
            seen.add(w.data_ptr())
            wbytes += w.numel() * w.element_size() * passes.get(id(mod), 1)
    for mod in expert_modules(ex):        # (each choice a different expert, as far as there are enough of them)
        wbytes += int(sum(p.numel() * p.element_size() for p in (mod.gate_up, mod.down)) * min(1.0, batch * mod.top / mod.experts))
    if ex.latents or ex.state_modules:    # cached rows seen by each attention layer; state read and written once
        kv = sum(batch * min(ctx_mid, m.window or ctx_mid) * m.row_cols * ex.dtype.itemsize for m in ex.model.modules()
                 if hasattr(m, "row_cols"))
        kv += sum(batch * min(ctx_mid, m.mask.window or ctx_mid) * 2 * m.num_kv_heads * m.head_dim * ex.dtype.itemsize
                  for m in ex.model.modules() if hasattr(m, "k_cache"))
        kv += sum(2 * batch * t.numel() // (2 * t.shape[1]) * t.element_size() for m in recurrent_modules(ex)
                  for t in (m.conv_state, m.ssm_state if hasattr(m, "ssm_state") else m.state))
        kv += sum(2 * batch * m.n * 4 for m in gru_modules(ex))
    else:
        L, nb, bs, hkv, d = ex.kv_cache.shape[1:]
        kv = L * batch * ctx_mid * 2 * hkv * d * ex.dtype.itemsize
    gbs = (wbytes + kv) / (ms_per_step * 1e-3) / 1e9
    return {"bound": "hbm", "weight_bytes_per_gpu": wbytes, "kv_bytes_per_step_per_gpu": int(kv),
            "bytes_per_step_per_gpu": int(wbytes + kv), "achieved": round(gbs, 1), "peak": HBM_PEAK_GBS, "unit": "GB/s",
            "frac": round(gbs / HBM_PEAK_GBS, 4), "mean_context": ctx_mid}


def recurrent_modules(ex) -> list:
    return [m for m in ex.state_modules if hasattr(m, "conv_state")]


def gru_modules(ex) -> list:
    return [m for m in ex.state_modules if type(m).__name__ == "MinGRU"]


def expert_modules(ex) -> list:
    return [m for m in ex.model.modules() if type(m).__name__ == "ExpertMLP"]


def release_all(engine):
    """Drop every queued / running sequence and give its blocks back (between two records on one engine)."""
    sch = engine.scheduler
    for seq in list(sch.running) + ([sch.prefilling] if sch.prefilling is not None else []):
        sch.block_manager.deallocate(seq)
    sch.running.clear()
    sch.waiting.clear()
    sch.prefilling = None
    ex = engine.model_runner.inference_executor
    ex.speculate_next = False
    drop = getattr(ex, "_drop_speculation", None)
    if drop is not None:
        drop()
    torch.cuda.synchronize()


def prefill_flops(heads: int, head_dim: int, lens, chunk: int = 0, window: int = 0) -> int:
    """Causal flash prefill without a cached prefix, one layer (K2): sum over sequences of
    4 H D (Sq Sk - Sq (Sq - 1) / 2) with Sq = Sk = len; a chunk mask cuts a sequence into pieces of ``chunk`` tokens; a window counts its pairs."""
    if window:
        return 4 * heads * head_dim * sum(min(i + 1, window) for n in lens for i in range(n))
    if chunk:
        lens = [m for n in lens for m in [chunk] * (n // chunk) + [n % chunk]]
    return sum(4 * heads * head_dim * (n * n - n * (n - 1) // 2) for n in lens)


def _mfma_busy_quote():
    for name in ("r04_pmc_prefill.json", "r03_pmc_prefill.json"):
        path = os.path.join(ROOT, "profiles", name)
        if os.path.exists(path):
            with open(path) as f:
                for key, rec in json.load(f).items():
                    if isinstance(rec, dict) and "mfma_utilisation" in rec:
                        return rec["mfma_utilisation"], f"profiles/{name}: {key.split(' (')[0]} -- SQ_VALU_MFMA_BUSY_CYCLES / (1024 SIMDs x GRBM_GUI_ACTIVE / 8), rocprofv3 --pmc in a pass of its own (counters cannot be read inside a timed run)"
    return None, None


def prefill_records(engine, model, gpus=1, cases=PREFILL_CASES, reps=5):
    """Prefill tokens/s of the whole model step (config-4 prompt shapes): n prompts x len fresh
    random tokens through ``execute_batch(prefill=True)`` -- input build, H2D, every layer, LM head on the last
    tokens, sampler, D2H of the n tokens.  One warm-up per shape, then the median of ``reps`` timed batches; then ONE more
    batch whose mv_prefill_varlen launches (one per layer) are bracketed by HIP event pairs -> ``roofline``."""
    from minivllm_amd import hip_ops
    from minivllm_amd.engine.sequence import Sequence
    from minivllm_amd.layers import attention as attn_mod

    ex, bm = engine.model_runner.inference_executor, engine.scheduler.block_manager
    cfgm = MODELS[model]
    vocab = cfgm["vocab_size"]
    heads = cfgm["num_attention_heads"] // gpus
    head_dim = cfgm.get("head_dim") or cfgm["hidden_size"] // cfgm["num_attention_heads"]
    busy, busy_src = _mfma_busy_quote()
    g = torch.Generator().manual_seed(1)
    out = []
    latent = bool(ex.latents)
    entry = "latent_prefill" if latent else "prefill_varlen"
    for n, ln in cases:
        times, probe = [], _EventProbe()
        for rep in range(reps + 2):
            seqs = [Sequence(torch.randint(0, vocab, (ln,), generator=g).tolist(), block_size=64) for _ in range(n)]
            for s in seqs:
                bm.allocate(s)
            probing = rep == reps + 1
            entries = {entry: "prefill", "ssm_prefill": "ssm", "delta_prefill": "delta", "moe_linear": "experts", "gru_prefill": "gru",
                       "stream_update": "edges", "residual_update": "edges", "gelu_erf": "act", "act_and_mul": "act"}
            reals = {e: getattr(hip_ops, e) for e in entries}
            if probing:
                for e, key in entries.items():
                    setattr(attn_mod.hip_ops, e, probe.wrap(key, reals[e]))
            try:
                torch.cuda.synchronize()
                t0 = time.perf_counter()
                ex.execute_batch(seqs, prefill=True)
                torch.cuda.synchronize()
                dt = time.perf_counter() - t0
            finally:
                for e, real in reals.items():
                    setattr(attn_mod.hip_ops, e, real)
            for s in seqs:
                bm.deallocate(s)
            if rep and not probing:
                times.append(dt)
        med = statistics.median(times)
        t_us = probe.times_us("prefill")
        m = statistics.median(t_us)
        kept = [t for t in t_us if t <= 3 * m]
        us = sum(kept) / len(kept)
        if latent:     # expanded form: scores over dim + rot columns, values of vdim columns, keys inside the window
            m0 = next(m for m in ex.model.modules() if hasattr(m, "row_cols"))
            seen = n * sum(min(i + 1, m0.window or ln) for i in range(ln))
            flops = seen * m0.heads * 2 * (m0.dq + m0.dv)
        else:
            flops = prefill_flops(heads, head_dim, [ln] * n, cfgm.get("chunk", 0), cfgm.get("window", 0))
        tf = flops / us / 1e6
        out.append({"metric": "prefill tokens/s", "model": model, "tp": gpus, "prompts": n, "prompt_len": ln,
                    "batches_timed": reps, "warmup_batches": 1, "ms_per_batch": round(med * 1e3, 3),
                    "value": round(n * ln / med, 1), "unit": "tokens/s",
                    "timing": "wall clock around execute_batch(prefill=True) bracketed by torch.cuda.synchronize(), median",
                    "roofline": {"bound": "mfma", "kernel": "latent_prefill_kernel" if latent else "prefill_mfma_kernel", "achieved": round(tf, 1),
                                 "peak": MFMA_PEAK_TFLOPS, "unit": "TFLOP/s", "frac": round(tf / MFMA_PEAK_TFLOPS, 4),
                                 "traffic": None, "flops_per_launch": flops, "us_per_launch": round(us, 2),
                                 "launches_timed": len(kept), "heads_per_rank": heads,
                                 "share_of_step": round(us * len(t_us) / (med * 1e6), 4),
                                 "mfma_busy": busy, "mfma_busy_source": busy_src,
                                 "timing": f"HIP event pairs around every mv_{entry} launch of one extra (untimed) batch, on the launching stream"}})
        out[-1].update(_edge_prefill(ex, n * ln, probe))
        if gru_modules(ex):
            m0, us = gru_modules(ex)[0], statistics.median(probe.times_us("gru"))
            out[-1]["ssm_roofline"] = dict(_hbm(n * ln * m0.n * 4 * ex.dtype.itemsize, us), kernel="gru_chunk_kernel + gru_walk_kernel")
            out[-1].update(_delta_and_expert_prefill(ex, n * ln, probe))
        elif recurrent_modules(ex) and hasattr(recurrent_modules(ex)[0], "state"):
            out[-1].update(_delta_and_expert_prefill(ex, n * ln, probe))
        elif ex.state_modules:
            m0, t_ssm = ex.state_modules[0], sorted(probe.times_us("ssm"))
            us = t_ssm[len(t_ssm) // 2]
            byt = n * ln * (2 * m0.heads * m0.p + 2 * m0.groups * m0.n + m0.heads) * ex.dtype.itemsize
            out[-1]["ssm_roofline"] = {"bound": "hbm", "kernel": "ssm_chunk_kernel", "bytes_per_launch": byt, "us_per_launch": round(us, 2),
                                       "achieved": round(byt / us / 1e3, 1), "peak": HBM_PEAK_GBS, "unit": "GB/s",
                                       "frac": round(byt / us / 1e3 / HBM_PEAK_GBS, 4)}
    return out


def _hbm(byt: int, us: float) -> dict:
    return {"bound": "hbm", "bytes_per_launch": int(byt), "us_per_launch": round(us, 2), "achieved": round(byt / us / 1e3, 1),
            "peak": HBM_PEAK_GBS, "unit": "GB/s", "frac": round(byt / us / 1e3 / HBM_PEAK_GBS, 4)}


def _edge_prefill(ex, tokens: int, probe) -> dict:
    """The launches between two sublayers (layers of a mixer and a feed-forward each): behind the mixers, and behind the dense
    feed-forwards, as bytes of the stream(s) read and written, the sublayer's output and the next one's input; the activation kernel of
    the dense feed-forwards."""
    stack, out, item = getattr(ex.model, "stack", []), {}, ex.dtype.itemsize
    t = probe.times_us("edges") if stack and all(getattr(la, "mlp", None) is not None for la in stack) else []
    if len(t) == 1 + 2 * len(stack):
        w, n = ex.model.embed.shape[1], getattr(ex.model.config, "streams", 1)
        dense = [i for i, la in enumerate(stack) if not hasattr(la.mlp, "experts")][:-1]      # (not the last edge: it reads differently)
        for key, us in (("edge_roofline", t[1::2]), ("shift_edge_roofline" if n > 1 else "ff_edge_roofline", [t[2 + 2 * i] for i in dense])):
            if us:
                out[key] = _hbm(tokens * w * (8 * n + 2 * item), statistics.median(us))
        dense = next((la.mlp for la in stack if not hasattr(la.mlp, "experts")), None)
        acts = probe.times_us("act")
        if acts:
            lin = getattr(dense, "up", None)
            byt = 2 * lin.weight.shape[0] if lin is not None else 3 * (dense.gate_up.weight.shape[0] // 2)
            out["act_roofline"] = _hbm(tokens * byt * item, statistics.median(acts))
    return out


def _delta_and_expert_prefill(ex, tokens: int, probe) -> dict:
    """Rooflines of mv_delta_prefill (bytes of its inputs and outputs, the layers of each kind apart) and of the two expert products."""
    out, mods = {}, recurrent_modules(ex)
    t = probe.times_us("delta")
    for key, kind in (("ssm_roofline", False), ("channel_decay_roofline", True)):
        mine = [(m, us) for m, us in zip(mods, t) if m.shape.channel_decay == kind]
        if mine:
            s, us = mine[0][0].shape, statistics.median(u for _, u in mine)
            byt = tokens * (2 * s.heads * s.p + 2 * s.groups * s.n + s.heads * (1 + (s.n if kind else 1))) * ex.dtype.itemsize
            names = "delta_prepare_kernel + delta_walk_kernel" if kind else "delta_scalar_prepare_kernel + delta_scalar_walk_kernel"
            out[key] = {"bound": "hbm", "kernel": names, "bytes_per_launch": byt,
                        "us_per_launch": round(us, 2), "achieved": round(byt / us / 1e3, 1), "peak": HBM_PEAK_GBS, "unit": "GB/s",
                        "frac": round(byt / us / 1e3 / HBM_PEAK_GBS, 4)}
    experts, t = expert_modules(ex), probe.times_us("experts")
    if experts:
        m0 = experts[0]
        pairs = tokens * m0.top * m0.experts / m0.router.shape[0]      # (identity experts have no product)
        for key, us, n in (("gate_up", t[0::2], 2), ("down", t[1::2], 1)):
            us, flops = statistics.median(us), 2 * pairs * n * m0.f * m0.w
            out[f"expert_{key}_roofline"] = {"bound": "mfma", "kernel": "moe_tile_kernel", "flops_per_launch": int(flops),
                                             "us_per_launch": round(us, 2), "achieved": round(flops / us / 1e6, 1),
                                             "peak": MFMA_PEAK_TFLOPS, "unit": "TFLOP/s",
                                             "frac": round(flops / us / 1e6 / MFMA_PEAK_TFLOPS, 4)}
    return out


def timed_decode(engine, args, dist=None):
    """W untimed + exactly K timed engine decode steps, barrier + synchronize on both sides, max over ranks."""
    def barrier():
        torch.cuda.synchronize()
        if args.gpus > 1:
            dist.barrier()
            torch.cuda.synchronize()
    for _ in range(args.warmup):
        engine.step()
    barrier()
    t0 = time.perf_counter()
    for _ in range(args.steps):
        engine.step()
    barrier()
    elapsed = time.perf_counter() - t0
    if args.gpus > 1:
        t = torch.tensor([elapsed], dtype=torch.float64, device="cuda")
        dist.all_reduce(t, op=dist.ReduceOp.MAX)
        elapsed = float(t.item())
    assert len(engine.scheduler.running) == args.batch, "a sequence finished inside the timed region"
    return elapsed


def usable_cores() -> int:
    """CPU threads this process may really use: the affinity mask, cut by a cgroup CPU quota where one is set."""
    n = len(os.sched_getaffinity(0)) if hasattr(os, "sched_getaffinity") else (os.cpu_count() or 1)
    try:
        with open("/sys/fs/cgroup/cpu.max") as f:
            quota, period = f.read().split()
        if quota != "max":
            n = min(n, max(1, int(int(quota) / int(period))))
    except (OSError, ValueError):
        pass
    return n


def _cpu_threads() -> int:
    # torch's default is one thread per physical core of the HOST; a GPU box hands a job a share of the host
    # (16 CPUs for one GPU on this pool), and 128 threads time-sliced on that share is what made this baseline
    # swing 3.4x between two boxes in round 2
    n = max(1, min(torch.get_num_threads(), usable_cores()))
    torch.set_num_threads(n)
    return n


def cpu_baseline(args):
    """Oracle (CPU restatement of the reference's eager path) decode tokens/s, bounded sample: one untimed warm-up
    step, then ``--cpu-steps`` timed steps, median."""
    from oracle.model import OracleModel

    threads = _cpu_threads()
    cfg = MODELS[args.model]
    b, ctx = 8, 128
    nblk = -(-(ctx + 64) // 64)
    t_build = time.perf_counter()
    model = OracleModel.random(cfg, dtype=torch.float32, num_blocks=b * nblk, block_size=64)
    for kc, vc in zip(model.k_cache, model.v_cache):
        kc.normal_()
        vc.normal_()
    tables = torch.arange(b * nblk, dtype=torch.int32).view(b, nblk)
    lens = torch.full((b,), ctx, dtype=torch.int32)
    ids = torch.randint(0, cfg["vocab_size"], (b,))
    build_s = time.perf_counter() - t_build
    per_step = []
    for step in range(args.cpu_steps + 1):
        t0 = time.perf_counter()
        pos = (lens - 1).long()
        slots = (tables[torch.arange(b), (pos // 64)] * 64 + (pos % 64).int()).int()
        meta = dict(is_prefill=False, slot_mapping=slots, block_tables=tables, context_lens=lens)
        logits = model.forward_logits(ids, pos, meta)
        ids = logits.float().argmax(-1)
        lens = lens + 1
        if step:                             # step 0 is the warm-up (first touch of 6.9 GB of fp32 weights)
            per_step.append(time.perf_counter() - t0)
    med = statistics.median(per_step)
    return {"value": round(b / med, 2), "unit": "tokens/s", "cores": threads, "kind": "port",
            "sample": f"{args.model} fp32 (the reference's CPU dtype, examples/cpu_inference_opt.py:143-151) random weights, "
                      f"decode only, B={b}, ctx {ctx}->{ctx + len(per_step) + 1}: 1 untimed warm-up step, then the median of "
                      f"{len(per_step)} steps ({min(per_step):.2f}-{max(per_step):.2f} s per step; oracle/model.py; build "
                      f"{build_s:.0f}s).  A bounded sample of the headline model, NOT the headline batch: the CPU path "
                      f"needs minutes per step at B={args.batch}, ctx {args.ctx}; tokens/s per sequence at B={b} is the "
                      f"CPU's best case (weights are re-read per step whatever B is).  cores = torch intra-op threads = "
                      f"min(torch's default, the CPUs this job may use: {usable_cores()}) of {os.cpu_count()} logical CPUs"}


OPT_125M = dict(model_type="opt", architectures=["OPTForCausalLM"], hidden_size=768, num_hidden_layers=12,
                num_attention_heads=12, ffn_dim=3072, vocab_size=50272, max_position_embeddings=2048,
                word_embed_proj_dim=768, do_layer_norm_before=True, activation_function="relu",
                enable_bias=True, layer_norm_elementwise_affine=True, tie_word_embeddings=True,
                torch_dtype="float16", eos_token_id=2, bos_token_id=2, pad_token_id=1)


def cpu_config1(reps=3):
    """BASELINE config 1 on this host's CPU cores: the workload of the reference's examples/cpu_inference_opt.py
    (:56-62 five prompts, :143-158 max_num_seqs=8, max_model_len=1024, eager, fp32, temperature 0.6 / top_p 0.95 /
    top_k 40 / 50 new tokens) at the TRUE OPT-125M dimensions with random weights (no checkpoint offline), token-id
    prompts of 16 tokens (what those prompts come to under the chat template), through the build's host engine
    (scheduler, block manager, input builder) with the CPU restatement of the eager model as its runner."""
    from minivllm_amd import Config, SamplingParams
    from minivllm_amd.engine.input_builder import InputBuilder
    from minivllm_amd.engine.llm_engine import LLMEngine
    from oracle.model import OracleModel, OracleRunner

    threads = _cpu_threads()
    with tempfile.TemporaryDirectory() as workdir:
        with open(os.path.join(workdir, "config.json"), "w") as f:
            json.dump(OPT_125M, f)
        cfg = Config(workdir, dtype="float32", max_num_seqs=8, max_model_len=1024, max_num_batched_tokens=1024,
                     enforce_eager=True, kvcache_block_size=64, num_kvcache_blocks=8 * 16, load_format="dummy", seed=0)
        model = OracleModel.random(OPT_125M, dtype=torch.float32, num_blocks=cfg.num_kvcache_blocks, block_size=64)
        g = torch.Generator().manual_seed(0)
        prompts = [torch.randint(3, OPT_125M["vocab_size"], (16,), generator=g).tolist() for _ in range(5)]
        sp = SamplingParams(temperature=0.6, top_p=0.95, top_k=40, max_tokens=50, ignore_eos=True)
        runs = []
        for rep in range(reps + 1):
            engine = LLMEngine(cfg, model_runner=OracleRunner(model, InputBuilder(64, 8, 1024, cfg.max_num_batched_tokens), seed=rep))
            t0 = time.perf_counter()
            outs = engine._generate_local(prompts, sp, use_tqdm=False)
            dt = time.perf_counter() - t0
            n = sum(len(o["token_ids"]) for o in outs)
            assert n == 5 * 50
            if rep:
                runs.append(n / dt)
    return {"value": round(statistics.median(runs), 1), "unit": "tokens/s", "cores": threads, "kind": "port",
            "sample": f"BASELINE config 1: OPT-125M fp32 at its true dimensions (random weights), 5 prompts x 16 token ids, 50 "
                      f"new tokens each, temperature 0.6 / top_p 0.95 / top_k 40 (reference examples/cpu_inference_opt.py:"
                      f"143-158), generated tokens / wall time of generate() incl. the prefill step; 1 untimed warm-up run, "
                      f"then the median of {len(runs)} runs ({min(runs):.1f}-{max(runs):.1f}); host engine of this build + "
                      f"oracle/model.py as its runner.  The reference itself measured 28.6 tokens/s (BASELINE.md) and the "
                      f"survey container 120.6 tokens/s on 8 threads with the real checkpoint"}


def _tp_info(engine, args, model, ar_probe, dist):
    """(N > 1) what the process group is, which all-reduce ran, per-rank all-reduce probe, and the proof that every rank
    generated the same tokens (SPMD lock-step): a digest of all sequences compared across ranks."""
    import hashlib

    from minivllm_amd import parallel_state
    from minivllm_amd.custom_allreduce import describe_status

    world = args.gpus
    ar = parallel_state.get_custom_all_reduce()
    words = ar.status_words() if ar is not None else None
    allreduce = "rccl" if ar is None else (
        f"p2p two-shot kernel (validated against the backend at start-up, {ar.calls} calls)"
        if words[0] == 0 else f"p2p two-shot kernel: RESULT INVALID, {describe_status(words)}")
    group = engine.model_runner.distributed_manager.control_group
    digest = hashlib.sha256(json.dumps([s.completion_token_ids for s in engine.scheduler.running]).encode()).hexdigest()
    digests = [None] * world
    dist.all_gather_object(digests, digest, group=group)
    assert len(set(digests)) == 1, f"ranks generated different tokens: {digests}"
    probes = [None] * world
    dist.all_gather_object(probes, ar_probe, group=group)
    # what the process group actually is: backend "nccl" = RCCL on ROCm, and how many ranks it spans
    info = {"backend": dist.get_backend(), "ranks": dist.get_world_size(),
            "activation_all_reduce": "rccl" if ar is None else "p2p",
            "all_reduces_per_step": 2 * MODELS[model]["num_hidden_layers"] + 1,
            "logit_exchange": "per-rank argmax merge (greedy batch): no [B, V/tp] all-gather",
            "tokens_identical_on_all_ranks": True, "allreduce_probe_per_rank": probes}
    return allreduce, info


def decode_record(engine, args, model, dist, sampling=None, seed=0, probes=True):
    """One decode record on a filled engine: timed steps, attention roofline (+ all-reduce probe), projection roofline,
    whole-step roofline, and under TP the token digest.  ``args`` carries batch / ctx / steps / warmup of THIS record."""
    note(f"{model} tp{args.gpus} B={args.batch} ctx={args.ctx} {'sampled' if sampling else 'greedy'}: prefill of the prompts")
    prefill_tps = fill_prompts(engine, args, model, sampling=sampling, seed=seed)
    note("  timed decode steps")
    elapsed = timed_decode(engine, args, dist)
    ms = elapsed / args.steps * 1e3
    ex = engine.model_runner.inference_executor
    graphs = bool(ex.graphs or ex.greedy_graphs)
    rec = {"metric": "decode tokens/s", "model": model, "tp": args.gpus, "value": round(args.batch * args.steps / elapsed, 1),
           "unit": "tokens/s", "steps": args.steps, "warmup": args.warmup, "ms_per_step": round(ms, 4), "dtype": "bf16",
           "config": {"workload": f"{model} decode, B={args.batch}, ctx={args.ctx}, kvcache_block_size=64, max_num_seqs={args.batch}, "
                                  f"{'hipGraph' if graphs and not args.eager else 'eager'} decode, "
                                  + (f"sampled (temperature {sampling['temperature']}, top_p {sampling['top_p']}, top_k {sampling['top_k']}: "
                                     f"reference examples/cpu_inference_opt.py:153-158)" if sampling else "greedy"),
                      "parallelism": f"tp{args.gpus}", "kv_blocks": engine.config.num_kvcache_blocks,
                      "max_model_len": engine.config.max_model_len}}
    if not probes:
        return rec, prefill_tps
    note("  attention roofline probe (eager steps)")
    roof, ar_probe = decode_roofline(engine, args, model)
    rec["roofline"] = roof
    rec["step_roofline"] = step_roofline(engine, model, args.batch, args.ctx + args.warmup + args.steps // 2, ms)
    if args.gpus > 1:
        allreduce, info = _tp_info(engine, args, model, ar_probe, dist)
        rec["config"]["allreduce"], rec["config"]["tensor_parallel"] = allreduce, info
    return rec, prefill_tps


def run_records(args, workdir, dist):
    """Execute ``record_plan``: one engine per model, records in plan order.  Every rank runs the same sequence (SPMD)."""
    import gc

    plan = record_plan(args.gpus, args.model, args.batch, args.ctx)
    if args.rehearse_n8:
        # the N = 8 flow (rejection, then a third engine with the 72B layer shape) on what two ranks on one card can hold
        odd = dict(MODELS["qwen2-7b"], num_attention_heads=7, num_key_value_heads=1, hidden_size=896, num_hidden_layers=2)
        MODELS["qwen2-7b-odd-heads (rehearsal)"] = odd
        MODELS["qwen2-72b-4-layers (rehearsal)"] = dict(MODELS["qwen2-72b"], num_hidden_layers=4)
        plan = [plan[0], dict(kind="rejected", model="qwen2-7b-odd-heads (rehearsal)", tp=args.gpus),
                dict(kind="decode", model="qwen2-72b-4-layers (rehearsal)", tp=args.gpus, batch=256, ctx=1024, sampling="greedy",
                     max_model_len=4096)]
    if args.no_secondary or args.synthetic_kv:
        plan = plan[:1]
    records, engine, engine_model, engine_args, first_on_engine = [], None, None, None, True
    headline_prefill_tps = None
    for i, item in enumerate(plan):
        model = item["model"]
        headline = bool(item.get("headline"))
        if item["kind"] == "rejected":
            if engine is not None:
                engine.exit()
                engine, engine_model = None, None
                gc.collect()
                torch.cuda.empty_cache()
            note(f"{model} tp{item['tp']}: expecting the reference's rejection")
            a2 = argparse.Namespace(**vars(args))
            a2.model, a2.batch, a2.ctx = model, 256, 1024
            try:
                eng = build_engine(a2, os.path.join(workdir, f"{model}-rejected"), model)
            except ValueError as e:
                records.append({"metric": "decode tokens/s", "model": model, "tp": item["tp"], "value": None,
                                "status": "rejected, as in reference", "error": f"ValueError: {e}",
                                "reference": "minivllm/models/qwen_base.py:95-104 (q / kv heads must divide by the TP degree: "
                                             f"{MODELS[model]['num_attention_heads']} / {MODELS[model]['num_key_value_heads']} by "
                                             f"{item['tp']}); the build raises the same error instead of silently replicating KV heads"})
            else:
                eng.exit()
                raise AssertionError(f"{model} at TP={item['tp']} was accepted: the reference rejects it")
            continue
        if engine_model != model:
            if engine is not None:
                engine.exit()
                del engine
                gc.collect()
                torch.cuda.empty_cache()
            a2 = argparse.Namespace(**vars(args))
            if not headline:
                a2.model, a2.batch, a2.ctx = model, item.get("batch", 256), item.get("ctx", 1024)
                a2.steps, a2.warmup = max(20, min(args.steps, 64)), max(5, min(args.warmup, 8))
                if args.gpus > 1:
                    # the secondary TP engines capture only the bucket this workload replays (each bucket x 3 graph
                    # families x up to 80 layers is seconds of start-up the driver's clock would pay 21 times over)
                    os.environ["MV_GRAPH_BATCH_SIZES"] = str(a2.batch)
            note(f"building {model} tp{args.gpus}" + (" (KV pool from free HBM)" if item.get("auto_kv") or args.auto_kv else ""))
            engine = build_engine(a2, os.path.join(workdir, model), model, max_model_len=item.get("max_model_len"),
                                  auto_kv=item.get("auto_kv"))
            os.environ.pop("MV_GRAPH_BATCH_SIZES", None)
            engine_model, engine_args, first_on_engine = model, a2, True
        if item["kind"] == "decode":
            if not first_on_engine:
                release_all(engine)
            sampling = SAMPLED if item["sampling"] == "sampled" else None
            rec, tps = decode_record(engine, engine_args, model, dist, sampling=sampling, seed=0 if first_on_engine else 2,
                                     probes=sampling is None)
            if sampling is None and engine_args.batch > 16:
                note("  projection roofline (graph replays)")
                release_all(engine)
                rec["projection_roofline"] = projection_roofline(engine, engine_args.batch)
            else:
                release_all(engine)
            if item.get("auto_kv"):
                ex = engine.model_runner.inference_executor
                L, nb, bs, hkv, d = ex.kv_cache.shape[1:]
                rec["config"]["kv_pool_per_gpu"] = {
                    "blocks": nb, "block_bytes": 2 * L * bs * hkv * d * ex.dtype.itemsize,
                    "GiB": round(ex.kv_cache.numel() * ex.dtype.itemsize / 2 ** 30, 2), "local_kv_heads": hkv,
                    "sizing": "min((total*0.9 - used - peak + current) // block_bytes, max_num_seqs * ceil(max_model_len / 64)), "
                              "MIN over the ranks (reference inference_executor.py:245-318 with the LOCAL kv-head count)"}
            if headline:
                rec["headline"], headline_prefill_tps = True, tps
            records.append(rec)
            first_on_engine = False
        elif item["kind"] == "prefill":
            if not first_on_engine:
                release_all(engine)
            note(f"{model} tp{args.gpus} prefill {item['prompts']} x {item['prompt_len']}")
            records += prefill_records(engine, model, args.gpus, cases=((item["prompts"], item["prompt_len"]),))
            first_on_engine = False
    if engine is not None:
        engine.exit()
    return records, headline_prefill_tps


def init_process_group(args):
    """(N > 1) ONE process group for the whole run, made here and not by the first engine: engines come and go (one per
    model of the plan) and the DistributedManager only destroys a group it made itself."""
    import torch.distributed as dist

    backend = os.environ.get("MINIVLLM_TP_BACKEND", "nccl")
    rank, world = int(os.environ["RANK"]), int(os.environ["WORLD_SIZE"])
    kw = {}
    local = int(os.environ.get("LOCAL_RANK", rank)) % torch.cuda.device_count()
    torch.cuda.set_device(local)
    if backend == "nccl":
        kw["device_id"] = torch.device("cuda", local)
    from datetime import timedelta

    dist.init_process_group(backend=backend, rank=rank, world_size=world, timeout=timedelta(minutes=10), **kw)
    return dist


def attention_graph_roofline(engine, model) -> tuple:
    """-> (attention, state space step or None).  The decode attention launches of one step (every layer run, on the running batch's tables, lengths and K/V planes, query
    rows random) captured into a graph and replayed.  A design's small batches are launch-bound when run eagerly: event pairs
    around its launches would time the host."""
    from minivllm_amd import hip_ops
    from minivllm_amd.utils.context import get_context, reset_context

    ex = engine.model_runner.inference_executor
    seqs = list(engine.scheduler.running)
    ex._drop_speculation()
    torch.cuda.synchronize()
    ex._ship_decode(ex.builder.decode(seqs))
    ctx = get_context()
    tables, lens, slots = ctx.block_tables, ctx.context_lens, ctx.state_slots
    reset_context()
    if ex.latents:
        return _latent_graph_roofline(ex, tables, lens), _state_graph_roofline(ex, lens, slots)
    mods = [m for m in ex.model.modules() if hasattr(m, "k_cache") and hasattr(m, "v_cache")]
    m0 = mods[0]
    q = torch.randn((len(seqs), m0.num_heads, m0.head_dim), device=ex.device).to(ex.dtype)
    gate = torch.randn_like(q).flatten(1) if type(ex.model).__name__ == "SemezenForCausalLM" else None

    def run():
        for m in mods:
            hip_ops.paged_decode(q, m.k_cache, m.v_cache, tables, lens, m.scale, chunk=m.chunk, mask=m.gated(gate))
    us = _graph_time_us(run, len(mods))
    seen = [n - (n - 1) // m0.chunk * m0.chunk if m0.chunk else n for n in lens.tolist()]
    if m0.mask and m0.mask.window:
        seen = [min(n, m0.mask.window + m0.mask.keep_first) for n in seen]
    algo = (sum(seen) * 2 * m0.num_kv_heads * m0.head_dim + (2 if gate is None else 3) * q.numel()) * ex.dtype.itemsize
    return {"bound": "hbm", "achieved": round(algo / us / 1e3, 1), "peak": HBM_PEAK_GBS, "unit": "GB/s",
            "frac": round(algo / us / 1e3 / HBM_PEAK_GBS, 4), "bytes_per_launch": algo, "us_per_launch": round(us, 2),
            "timing": f"{len(mods)} launches (split-KV combine included) captured into a hipGraph, median of 5 replays / launches"}, (
                _gru_graph_roofline(ex, lens, slots) if gru_modules(ex) else _delta_graph_roofline(ex, lens, slots) if recurrent_modules(ex) else None)


def _graph_roofline(byt: int, us: float, launches: int) -> dict:
    return {"bound": "hbm", "achieved": round(byt / us / 1e3, 1), "peak": HBM_PEAK_GBS, "unit": "GB/s",
            "frac": round(byt / us / 1e3 / HBM_PEAK_GBS, 4), "bytes_per_launch": byt, "us_per_launch": round(us, 2),
            "timing": f"{launches} launches (merges included) captured into a hipGraph, median of 5 replays / launches"}


def _latent_graph_roofline(ex, tables, lens) -> dict:
    """mv_latent_decode of every attention layer on the running batch, query rows random."""
    from minivllm_amd import hip_ops

    mods = [m for m in ex.model.modules() if hasattr(m, "row_cols")]
    m0, b = mods[0], lens.numel()
    q = torch.randn((b, m0.heads, m0.row_cols), device=ex.device).to(ex.dtype)

    def run():
        for m in mods:
            hip_ops.latent_decode(q, m.owner.latent_cache, tables, lens, m.kv_cols, m.scale, m.window)
    us = _graph_time_us(run, len(mods))
    seen = sum(min(n, m0.window or n) for n in lens.tolist())
    return _graph_roofline((seen * m0.row_cols + q.numel() + b * m0.heads * m0.kv_cols) * ex.dtype.itemsize, us, len(mods))


def _state_graph_roofline(ex, lens, slots) -> dict:
    """mv_ssm_step of every state space layer on the running batch (a step that is run again gives the same state)."""
    from minivllm_amd import hip_ops

    mods, b = ex.state_modules, lens.numel()
    m0 = mods[0]
    z = torch.randn((b, m0.in_proj.weight.shape[0]), device=ex.device).to(ex.dtype)

    def run():
        for m in mods:
            hip_ops.ssm_step(z[:, m.x_off:m.x_off + m.channels], z[:, m.dt_off:m.dt_off + m.heads], m.conv, m.conv_b, m.dt_bias, m.A_log,
                             m.D, m.shape, m.conv_state, m.ssm_state, slots, lens)
    us = _graph_time_us(run, len(mods))
    byt = 2 * b * (m0.ssm_state[0, 0].numel() * 4 + m0.conv_state[0, 0].numel() * ex.dtype.itemsize)
    byt += b * (m0.channels + m0.heads + m0.heads * m0.p) * ex.dtype.itemsize
    return _graph_roofline(byt, us, len(mods))


def _gru_graph_roofline(ex, lens, slots) -> dict:
    """mv_gru_step of every such layer on the running batch (a step that is run again gives the same state)."""
    from minivllm_amd import hip_ops

    mods, b = gru_modules(ex), lens.numel()
    n = mods[0].n
    z = torch.randn((b, 3 * n), device=ex.device).to(ex.dtype)
    out = torch.empty((b, n), dtype=ex.dtype, device=ex.device)

    def run():
        for m in mods:
            hip_ops.gru_step(z[:, :n], z[:, n:2 * n], z[:, 2 * n:], m.state, slots, lens, out)
    return _graph_roofline(b * n * (8 + 4 * ex.dtype.itemsize), _graph_time_us(run, len(mods)), len(mods))


def edge_graph_us(engine, batch: int) -> float | None:
    """One launch between a feed-forward and the next mixer, on random rows inside a graph: streams with a token shift, or a normed
    residual stream."""
    from minivllm_amd import hip_ops

    ex = engine.model_runner.inference_executor
    stack, kind = getattr(ex.model, "stack", []), type(ex.model).__name__
    if kind not in ("SemezenForCausalLM", "PununexForCausalLM"):
        return None
    w, c = ex.model.embed.shape[1], ex.model.config
    y = torch.randn((batch, w), device=ex.device).to(ex.dtype)
    n, pos = getattr(c, "streams", 1), torch.ones((batch,), dtype=torch.int64, device=ex.device)
    x, new = (torch.randn((batch, n, w), device=ex.device) for _ in range(2))
    slots = torch.arange(batch, dtype=torch.int32, device=ex.device)

    def run():
        for a, b in zip(stack, stack[1:]):
            if kind == "SemezenForCausalLM":
                hip_ops.stream_update(n, b.norm1, 1e-6, x=x, x_out=new, y=y, mix=a.hc2.mix, out_w=a.hc2.write, in_w=b.hc1.read,
                                      shift=hip_ops.StreamShift(b.shift.share, b.shift.prev, pos, slots))
            else:
                hip_ops.residual_update(x[:, 0], y=y, y_norm_w=a.norm2, y_norm_b=a.norm2_b, y_scale=a.ls2, layer_norm=True, eps=1e-6,
                                        dtype=ex.dtype)
    return round(_graph_time_us(run, len(stack) - 1), 2)


def _delta_graph_roofline(ex, lens, slots) -> dict:
    """mv_delta_step of the layers with a decay per head on the running batch (a step that is run again gives the same state)."""
    from minivllm_amd import hip_ops

    mods, b = [m for m in recurrent_modules(ex) if not m.shape.channel_decay], lens.numel()
    m0, s = mods[0], mods[0].shape
    z = torch.randn((b, m0.columns), device=ex.device).to(ex.dtype)
    at, cols = m0.at, s.heads * s.p

    def run():
        for m in mods:
            hip_ops.delta_step(s, z[:, :s.channels], z[:, at["b"]:at["b"] + s.heads], z[:, at["a"]:at["a"] + s.heads], m.dt_bias, m.A_log,
                               m.conv, m.conv_state, m.state, slots, lens, z[:, at["g"]:at["g"] + cols], m.norm, m.gate)
    us = _graph_time_us(run, len(mods))
    byt = 2 * b * (m0.state[0, 0].numel() * 4 + m0.conv_state[0, 0].numel() * ex.dtype.itemsize)
    return _graph_roofline(byt + b * (s.channels + 2 * s.heads + 2 * cols) * ex.dtype.itemsize, us, len(mods))


def expert_graph_rooflines(engine, batch: int) -> dict | None:
    """Routing and the two expert products of every layer with experts, on random rows: weight bytes of the experts that were chosen."""
    from minivllm_amd import hip_ops

    ex = engine.model_runner.inference_executor
    mods = expert_modules(ex)
    if not mods:
        return None
    out, m0 = {}, mods[0]
    h = torch.randn((batch, m0.w), device=ex.device).to(ex.dtype)
    groups = [m.route(h)[1] for m in mods]
    used = statistics.mean(len({e for e in g.tiles[:, 0].tolist() if e >= 0}) for g in groups)
    zs = [torch.randn((batch * m.top, m.f), device=ex.device).to(ex.dtype) for m in mods]

    def gate_up():
        for m, g in zip(mods, groups):
            hip_ops.moe_linear(h, m.gate_up, m.f, g, m.act, gather=True, experts=m.experts, in_scale=g.weights)

    def down():
        for m, g, z in zip(mods, groups, zs):
            hip_ops.moe_linear(z, m.down, m.w, g, experts=m.experts)

    def route():
        for m in mods:
            m.route(h)
    for name, run, n in (("gate_up", gate_up, 2), ("down", down, 1)):
        out[name] = _graph_roofline(int(used * n * m0.f * m0.w * ex.dtype.itemsize), _graph_time_us(run, len(mods)), len(mods))
    out["route_and_group_us"] = round(_graph_time_us(route, len(mods)), 2)
    return out


def design_records(args, workdir) -> dict:
    """``--design``: for every size of the design and for its peer, decode at several batches and prefill, on one engine each."""
    import gc

    out = {}
    for name, like in DESIGNS[args.design].items():
        for model in (name, like):
            a = argparse.Namespace(**vars(args))
            a.model, a.batch, a.ctx = model, max(b for b, _ in DESIGN_DECODE), max(c for _, c in DESIGN_DECODE)
            os.environ["MV_GRAPH_BATCH_SIZES"] = ",".join(str(b) for b, _ in DESIGN_DECODE)
            note(f"building {model}")
            engine = build_engine(a, os.path.join(workdir, model), model)
            os.environ.pop("MV_GRAPH_BATCH_SIZES", None)
            recs = []
            for i, (batch, ctx) in enumerate(DESIGN_DECODE):
                a.batch, a.ctx = batch, ctx
                rec, _ = decode_record(engine, a, model, None, seed=i, probes=False)
                rec["roofline"], state = attention_graph_roofline(engine, model)
                if state is not None:
                    rec["state_roofline"] = state
                experts = expert_graph_rooflines(engine, batch)
                if experts is not None:
                    rec["expert_rooflines"] = experts
                rec["edge_us"] = edge_graph_us(engine, batch)
                rec["step_roofline"] = step_roofline(engine, model, batch, ctx + a.warmup + a.steps // 2, rec["ms_per_step"])
                recs.append(rec)
                release_all(engine)
            for n, ln in DESIGN_PREFILL:
                note(f"{model} prefill {n} x {ln}")
                recs += prefill_records(engine, model, cases=((n, ln),))
            engine.exit()
            del engine
            gc.collect()
            torch.cuda.empty_cache()
            out[model] = recs
    return out


def design_line(args, records: dict) -> dict:
    """The JSON line of ``--design``: value = decode tokens/s of the last (largest) size, the pairs beside each other."""
    pairs = []
    for name, like in DESIGNS[args.design].items():
        for mine, peer in zip(records[name], records[like]):
            what = (f"prefill {mine['prompts']} x {mine['prompt_len']}" if "prompts" in mine
                    else mine["config"]["workload"].split(" ", 1)[1].split(", kvcache")[0])
            pairs.append({"model": name, "peer": like, "workload": what, "tokens_per_s": [mine["value"], peer["value"]],
                          "ratio": round(mine["value"] / peer["value"], 4),
                          "attention_frac_of_peak": [mine["roofline"]["frac"], peer["roofline"]["frac"]],
                          "state_frac_of_peak": (mine.get("state_roofline") or mine.get("ssm_roofline") or {}).get("frac"),
                          "step_frac_of_hbm_peak": [(r.get("step_roofline") or {}).get("frac") for r in (mine, peer)]})
    last = list(DESIGNS[args.design])[-1]
    head = records[last][0]
    return {"metric": f"{args.design} decode tokens/s", "value": head["value"], "unit": "tokens/s", "n_gpus": 1, "steps": args.steps,
            "warmup": args.warmup, "ms_per_step": head["ms_per_step"], "higher_is_better": True, "scaling": "strong",
            "vs_baseline": None, "dtype": "bf16", "data": "synthetic", "config": head["config"], "pairs": pairs, "records": records}


def main():
    args = parse()
    if args.design:
        if args.gpus != 1:
            raise SystemExit("--design runs on one GPU")
        with tempfile.TemporaryDirectory() as workdir:
            print(json.dumps(design_line(args, design_records(args, workdir))))
        return
    if args.cpu_config1_only:
        print(json.dumps(cpu_config1()))
        return
    rank = int(os.environ.get("RANK", "0"))
    world = int(os.environ.get("WORLD_SIZE", "1"))
    if args.gpus > 1 and "WORLD_SIZE" not in os.environ:
        # started bare (the driver's `python3 bench.py --gpus N`): become the launcher.  Nothing in this process has
        # touched the GPU (importing torch does not), and the ranks are CHILD processes, never an exec of this one.
        env = dict(os.environ)
        env.setdefault("HSA_ENABLE_IPC_MODE_LEGACY", "0")
        env.setdefault("OMP_NUM_THREADS", str(max(1, usable_cores() // args.gpus)))
        proc = subprocess.run(launch_command(args), env=env)
        raise SystemExit(proc.returncode)
    if args.gpus > 1 and world != args.gpus:
        raise SystemExit(f"--gpus {args.gpus} but WORLD_SIZE={world}: launch with --nproc-per-node {args.gpus}")
    os.environ.setdefault("HSA_ENABLE_IPC_MODE_LEGACY", "0")
    dist = None
    if args.gpus > 1:
        os.environ.setdefault("MASTER_ADDR", "127.0.0.1")
        os.environ.setdefault("TORCHELASTIC_RUN_ID", "bench")
        dist = init_process_group(args)
    with tempfile.TemporaryDirectory() as workdir:
        records, prefill_tps = run_records(args, workdir, dist)
    if dist is not None:
        dist.barrier()
        dist.destroy_process_group()
    if rank != 0:
        return
    cpu = None
    if not args.no_cpu_baseline and args.gpus == 1:          # rank 0, N=1 only
        note("cpu baseline (oracle on the host cores)")
        cpu = cpu_baseline(args)
        cpu["config1"] = cpu_config1()
    head = records[0]
    line = {
        "metric": "decode tokens/s", "value": head["value"], "unit": "tokens/s", "n_gpus": args.gpus,
        "steps": args.steps, "warmup": args.warmup, "ms_per_step": head["ms_per_step"],
        "higher_is_better": True, "scaling": "strong", "vs_baseline": None, "dtype": "bf16", "data": "synthetic",
        "config": dict(head["config"], kv_sizing="from free HBM (auto: the default user path)" if args.auto_kv else "explicit",
                       prefill="synthetic KV" if args.synthetic_kv else "engine prefill"),
        # steady state first (the 16 x 1024 record of `secondary`); the fresh engine's own prefill of the B x ctx prompts,
        # which includes one-time lazy set-up, under its own name
        "prefill_tokens_per_s": next((s["value"] for s in records[1:] if s.get("metric") == "prefill tokens/s"
                                      and s.get("model") == args.model and s.get("prompts") == 16), None),
        "prefill_tokens_per_s_method": "steady state: median of 5 timed batches of 16 x 1024 fresh tokens after a warm-up batch "
                                       "(the matching `secondary` record; null when the secondary records are skipped)",
        "prefill_tokens_per_s_first_run": None if prefill_tps is None else round(prefill_tps, 1),
        "prefill_tokens_per_s_first_run_method": "the B x ctx prompt tokens of this run / wall time of the engine's prefill steps "
                                                 "(first steps of a fresh engine: includes one-time lazy set-up)",
        "roofline": head.get("roofline"), "projection_roofline": head.get("projection_roofline"),
        "step_roofline": head.get("step_roofline"), "cpu_baseline": cpu,
        "secondary": records[1:] or None,
        "multi_gpu_note": None if args.gpus == 1 else
        "strong scaling: the same B x ctx workload tensor-parallel over N GPUs; secondary carries the Qwen2-7B / Qwen2-72B part "
        "of BASELINE.json's metric for this N (record_plan)",
    }
    print(json.dumps(line))


if __name__ == "__main__":
    main()
