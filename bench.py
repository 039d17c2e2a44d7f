#!/usr/bin/env python
"""Headline benchmark: EventGPT-7B bf16 greedy decode tokens/s (+ event-prefill ms) at 1..8 GPUs.

Matches the reference's headline measurement (decode throughput 54.0 tok/s,
LLM prefill 66.2 ms @ 636 tokens, vision 5.9 ms/frame on an RTX 4090 --
feasible/benchmark_inference/BENCHMARK_1FRAME_VS_8FRAMES_20260124_193405.md:18-29):
EventGPT-7B (Vicuna-7B decoder + CLIP ViT-L/14-336 tower), bf16, batch 1,
greedy, 1 event frame -> 636-token multimodal prompt.

    python bench.py --gpus N --steps K --warmup W

A *step* is one decode step (one new token per stream).  Before the W warm-up steps the sequence is
decoded once for ``--settle-steps`` untimed steps (reported as ``settle_steps``; 0 switches it off) and then
started afresh: the device's memory clocks need 150-200 ms of sustained streaming to reach the state a
serving engine runs in, and a 20-step sample taken right after the compute-bound vision / prefill phases
measures the state before it (2.66 vs 2.60 ms per step; `benchmarks/bench_decode_steps.py` shows the switch).
The timed region is exactly the K steps after the W warm-up steps, bracketed by barrier + synchronize.

* N = 1: the single-GPU serving engine (``runtime/engine.py``).
* N > 1: one process per GPU over RCCL.  Started without a torchrun environment, this
  script launches the N ranks itself (``python -m torch.distributed.run``, before anything
  in this process touches a GPU) and relays rank 0's JSON line.  The default parallelism is
  tensor-parallel (``parallel/tp.py``): the SAME single stream is served by N GPUs -- strong
  scaling, every decode step crosses 64 all-reduces -- and ``value`` is its tokens/s.  The
  batched configuration (32 event streams on the same TP group) is measured in the same run
  and reported under ``tp_batch32``, and so are N independent replicas (``dp_replicas``: no
  communication in the step, the fabric-free bound), one data-parallel fine-tuning step of the 7B
  model through the sharded AdamW's reduce-scatter / all-gather (``dp_train``: projector and LoRA
  stage), prefill hiding with drafter and verifier on two GPUs (``sd_two_gpu``) and, last, the same
  tensor-parallel measurement on the in-tree one-shot / two-shot all-reduce (``tp_oneshot``: run as
  a child job of every rank on its own process group, at any width up to 8, because that collective
  has never crossed a real link; before it starts, the line as it stands is also written to stderr
  and to ``gpurun_out/bench_line_before_oneshot.json``).
  The extras share a time limit (``--extras-timeout``) after which the line is printed without them.  ``--parallelism dp`` (independent replicas, no
  communication in the step) is available but is never the default: its curve says nothing
  about the fabric.

The JSON line carries ``rccl_world_size`` (the result of an actual all-reduce of ones),
``graph_captured`` (False if the decode step fell back to eager launches) and
``tp_allreduce`` (``rccl`` or ``oneshot``), so a fallback cannot pass for the real thing.

Weights are random-initialised with the 7B architecture and the prompt is a synthetic event
stream (no checkpoints or datasets are reachable here).  Rank 0 prints exactly one JSON line.
"""
from __future__ import annotations

import argparse
import json
import os
import socket
import subprocess
import sys
import threading
import time

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

BASELINE_DECODE_TOK_S = 54.0
BASELINE_PREFILL_MS = 66.16
BASELINE_VISION_MS = 5.93


def parse_args(argv=None):
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=128)
    ap.add_argument("--warmup", type=int, default=16)
    ap.add_argument("--settle-steps", type=int, default=96,
                    help="untimed decode steps before the warm-up (a fresh start of the sequence follows): "
                         "brings the device's memory clocks to their steady state; 0 = none")
    ap.add_argument("--prompt-len", type=int, default=636,
                    help="multimodal prompt length (636 = 1 event frame: 578 event + 58 text)")
    ap.add_argument("--frames", type=int, default=1)
    ap.add_argument("--max-len", type=int, default=2048, help="KV-cache capacity per stream")
    ap.add_argument("--parallelism", choices=["tp", "dp"], default="tp",
                    help="multi-GPU mode: tp = one stream over N GPUs (strong scaling, default); "
                         "dp = N independent replicas (weak scaling, no communication)")
    ap.add_argument("--model", choices=["7b", "small"], default="7b")
    ap.add_argument("--no-graph", action="store_true")
    ap.add_argument("--batch", type=int, default=1,
                    help="event streams decoded together per engine (32 = the batched serving config)")
    ap.add_argument("--no-batch32", action="store_true",
                    help="multi-GPU tp runs: skip the additional 32-stream measurement")
    ap.add_argument("--no-dp-extra", action="store_true",
                    help="multi-GPU tp runs: skip the additional independent-replicas measurement")
    ap.add_argument("--no-oneshot-extra", action="store_true",
                    help="multi-GPU tp runs over RCCL: skip the additional run on the in-tree one-shot / two-shot "
                         "all-reduce (a child job per rank, so that nothing it does can cost the headline line)")
    ap.add_argument("--oneshot-extra-timeout", type=float, default=200.0, help="seconds the child job may take")
    ap.add_argument("--no-dp-train-extra", action="store_true",
                    help="multi-GPU tp runs: skip the data-parallel fine-tuning step (sharded AdamW over the group)")
    ap.add_argument("--no-sd-extra", action="store_true",
                    help="multi-GPU tp runs: skip prefill hiding with drafter and verifier on two GPUs")
    ap.add_argument("--extras-timeout", type=float, default=420.0,
                    help="multi-GPU tp runs: seconds the additional measurements may take after the headline one; "
                         "past it the line is printed without them and the process ends (0 = no limit)")
    ap.add_argument("--extras-stall", type=float, default=0.0, help=argparse.SUPPRESS)  # tests of the limit: idle first
    ap.add_argument("--nsplit", type=int, default=None, help="KV splits of the decode attention")
    ap.add_argument("--allreduce", choices=["rccl", "oneshot", "auto"], default=None,
                    help="tensor-parallel collective (default: EVGPT_TP_ALLREDUCE or rccl)")
    ap.add_argument("--weight-format", choices=["bf16", "nf4", "fp4"], default="bf16",
                    help="nf4/fp4: the reference's 4-bit rows (bitsandbytes load_in_4bit); not the headline config")
    ap.add_argument("--layered", default=None, metavar="SIZES",
                    help="instead of the headline: prefill and decode of a layered decoder beside a LLaMA decoder "
                         "of equal size, one JSON line per pass (1b, 7b or both with a comma); one GPU")
    ap.add_argument("--layered-design", choices=["nusitar", "zapipel"], default="nusitar", help="which layered decoder")
    ap.add_argument("--layered-only", choices=["both", "nusitar", "zapipel", "llama"], default="both",
                    help="measure one of the two models")
    ap.add_argument("--layered-pass", default=None, metavar="PASS",
                    help="one pass only, e.g. prefill:1x4096 or decode:8 (for profiling)")
    ap.add_argument("--rehearsal", action="store_true",
                    help="run the multi-rank flow on ONE GPU: every rank drives cuda:0 and the group is gloo "
                         "(host-copied collectives, no graphs); exercises the code path, measures nothing useful")
    ap.add_argument("--probe", action="store_true",
                    help="launcher check: every rank joins a CPU (gloo) group, all-reduces a one and rank 0 "
                         "prints the world size; no GPU is touched")
    return ap.parse_args(argv)


# ------------------------------------------------------------------ launcher
def _free_port() -> int:
    with socket.socket() as s:
        s.bind(("127.0.0.1", 0))
        return s.getsockname()[1]


def launch_command(n: int, argv, port: int):
    """The command that runs this script as ``n`` ranks of one node."""
    return [sys.executable, "-m", "torch.distributed.run", "--nnodes=1", f"--nproc-per-node={n}",
            "--master-addr", "127.0.0.1", "--master-port", str(port), os.path.abspath(__file__), *argv]


def launch_ranks(n: int, argv) -> int:
    """Start ``n`` fresh ranks as a child job and wait for it.  The parent never initialises a
    GPU (a process that has must not be replaced or forked into ranks)."""
    env = dict(os.environ)
    env.setdefault("HSA_ENABLE_IPC_MODE_LEGACY", "0")
    env.setdefault("OMP_NUM_THREADS", "4")
    env["EVGPT_BENCH_CHILD"] = "1"
    return subprocess.call(launch_command(n, list(argv), _free_port()), env=env)


def probe_main(args) -> None:
    import torch
    import torch.distributed as dist
    os.environ.setdefault("MASTER_ADDR", "127.0.0.1")
    world = int(os.environ.get("WORLD_SIZE", "1"))
    rank = int(os.environ.get("RANK", "0"))
    if world > 1:
        dist.init_process_group("gloo")
        t = torch.ones(1)
        dist.all_reduce(t)
        seen = int(t.item())
    else:
        seen = 1
    if rank == 0:
        print(json.dumps({"probe": True, "n_gpus": world, "rccl_world_size": seen, "requested": args.gpus,
                          "scaling": "strong" if (args.parallelism == "tp" and world > 1) else "weak"}), flush=True)
    if world > 1:
        dist.destroy_process_group()


_CHILDREN = []      # child jobs of this rank that may still run


def kill_children() -> None:
    """End every child job of this rank, its whole process group (the child is a session leader)."""
    import signal
    for proc in list(_CHILDREN):
        if proc.poll() is None:
            try:
                os.killpg(proc.pid, signal.SIGKILL)
            except (ProcessLookupError, PermissionError):
                pass


def oneshot_child_command(args, world: int):
    """This script again, as one rank of a second job of the same size whose tensor-parallel engine
    asks for the in-tree all-reduce (``auto``: taken if its self-test passes, RCCL otherwise)."""
    cmd = [sys.executable, os.path.abspath(__file__), "--gpus", str(world), "--steps", str(args.steps),
           "--warmup", str(args.warmup), "--prompt-len", str(args.prompt_len), "--frames", str(args.frames),
           "--max-len", str(args.max_len), "--model", args.model,
           # (a gloo group only bootstraps the exchange of handles: there the mode is asked for outright)
           "--allreduce", "oneshot" if args.rehearsal else "auto",
           "--no-dp-extra", "--no-oneshot-extra", "--no-dp-train-extra", "--no-sd-extra",
           # its only extra is the 32-stream run: a 7B build + engine + run fits well inside this
           "--extras-timeout", str(max(60, int(args.oneshot_extra_timeout * 0.6))),
           "--settle-steps", str(args.settle_steps)]
    if args.rehearsal:
        cmd.append("--rehearsal")
    if args.no_graph:
        cmd.append("--no-graph")
    if args.no_batch32:
        cmd.append("--no-batch32")
    return cmd


def run_oneshot_child(args, dist, rank: int, world: int, local_rank: int, dev):
    """The in-tree all-reduce over IPC-mapped peer buffers has only ever run between processes
    that share one GPU.  Its first run across real links happens in a child process of every
    rank -- its own job and process group on another port -- so that a fault there ends the child,
    not the rank that holds the headline measurement.  Returns what rank 0's child measured."""
    import torch
    on_host = dist.get_backend() == "gloo"
    port = torch.tensor([_free_port() if rank == 0 else 0], dtype=torch.int64, device="cpu" if on_host else dev)
    dist.broadcast(port, 0)
    env = {k: v for k, v in os.environ.items() if not k.startswith("TORCHELASTIC_")}
    env.update({"MASTER_ADDR": "127.0.0.1", "MASTER_PORT": str(int(port.item())), "RANK": str(rank),
                "WORLD_SIZE": str(world), "LOCAL_RANK": str(local_rank), "LOCAL_WORLD_SIZE": str(world),
                "EVGPT_BENCH_CHILD": "1"})
    # its own session: on a time-out -- here or in the extras' watchdog -- the whole group of the child is
    # killed, so nothing of it keeps holding a GPU after this process has gone
    proc = subprocess.Popen(oneshot_child_command(args, world), env=env, stdout=subprocess.PIPE,
                            stderr=subprocess.PIPE, text=True, start_new_session=True)
    _CHILDREN.append(proc)
    try:
        stdout, stderr = proc.communicate(timeout=args.oneshot_extra_timeout)
    except subprocess.TimeoutExpired:
        kill_children()
        stdout, stderr = proc.communicate()
        if rank != 0:
            return None
        return {"error": f"child job not finished within {args.oneshot_extra_timeout} s"}
    finally:
        if proc in _CHILDREN and proc.poll() is not None:
            _CHILDREN.remove(proc)
    if rank != 0:
        return None
    lines = [l for l in stdout.splitlines() if l.startswith("{")]
    if proc.returncode != 0 or not lines:
        return {"error": f"child job ended with status {proc.returncode}: {stderr.strip()[-160:]}"}
    got = json.loads(lines[-1])
    out = {"tokens_per_s": got["value"], "ms_per_step": got["ms_per_step"], "tp_allreduce": got["tp_allreduce"],
           "graph_captured": got["graph_captured"], "event_prefill_ms": got["event_prefill_ms"]}
    if "tp_batch32" in got:
        out["tp_batch32"] = got["tp_batch32"]
    return out


# --------------------------------------------------------------------- bench
def layered_main(args) -> None:
    from eventgpt_amd.benchmarks import layered_bench
    kw = {}
    if args.layered_pass:
        kind, _, what = args.layered_pass.partition(":")
        kw = dict(prompts=(), packs=(), streams=())
        if kind == "decode":
            kw["streams"] = (int(what),)
        else:
            b, n = (int(v) for v in what.split("x"))
            kw.update({"prompts": (n,)} if b == 1 else {"packs": ((b, n),)})
    layered_bench.run(sizes=tuple(args.layered.split(",")), only=args.layered_only, design=args.layered_design, emit=lambda s: print(s, flush=True), **kw)


def build_model(args, dev):
    import torch
    from eventgpt_amd.models import ClipVisionConfig, EventChatConfig, EventChatModel
    if args.model == "7b":
        cfg = EventChatConfig.eventgpt_7b(vocab_size=32003)
        name = "EventGPT-7B (Vicuna-7B + CLIP ViT-L/14-336, random init)"
    else:
        cfg = EventChatConfig(vocab_size=32003, hidden_size=1024, intermediate_size=2816,
                              num_hidden_layers=4, num_attention_heads=8,
                              mm_visual_tower="small", event_feature_adaptor=True)
        cfg.vision_config = ClipVisionConfig(hidden_size=256, intermediate_size=1024,
                                             num_hidden_layers=2, num_attention_heads=4)
        name = "small-debug"
    model = EventChatModel.from_config(cfg, torch.bfloat16, dev, seed=1234)
    return cfg, model, name


def build_engine(args, model, dist, tp: bool, batch: int):
    ekw = {} if args.nsplit is None else {"nsplit": args.nsplit}
    if args.weight_format != "bf16":
        ekw["weight_format"] = args.weight_format
    budget = max(args.steps + args.warmup, args.settle_steps) + 8
    # the cache holds the prompt and every token of the run, whatever --steps asks for
    need = args.prompt_len + budget + 64
    max_len = max(args.max_len, (need + 255) // 256 * 256)
    if tp or batch > 1:
        from eventgpt_amd.parallel.tp import TensorParallelEngine
        return TensorParallelEngine(model, dist.group.WORLD if tp else None, max_len=max_len,
                                    max_batch=batch, max_new_tokens=budget, use_graph=not args.no_graph,
                                    allreduce=args.allreduce, **ekw)
    return model.engine(max_len=max_len, max_new_tokens=budget, use_graph=not args.no_graph, **ekw)


def timed_decode(args, engine, embeds, batch: int, dist, dev):
    """W warm-up steps, then exactly K timed steps bracketed by barrier + synchronize; MAX over ranks."""
    import torch

    def sync_all():
        if dist is not None:
            dist.barrier()
        torch.cuda.synchronize()

    engine.eos = -1

    def start():
        engine.reset()
        if batch == 1:
            engine.prefill(embeds)
        else:
            engine.prefill_batch([embeds] * batch)

    # Settling (untimed, reported as ``settle_steps``): the device's memory clocks take 150-200 ms of
    # sustained streaming to reach their steady state -- decode steps measured from an event after every
    # replay run at 2.68 ms for the first ~65 steps after compute-bound work (vision, prefill) and at 2.59 ms
    # from then on (`benchmarks/bench_decode_steps.py`).  A serving engine lives in the second state, and the
    # reference's figure is an average over whole generations, so the sequence is decoded once for
    # ``--settle-steps`` steps, then started again for the W warm-up steps and the K timed ones.
    cold_ms = None
    if args.settle_steps > 0:
        start()
        engine.decode_step(True)        # (captures the step's graph, outside every clock)
        start()
        # the unsettled figure, for the record: the first steps after the prefill, as a run without the
        # settling phase would time them (they are the start of that phase, not additional work)
        n_cold = min(20, args.settle_steps)
        sync_all()
        t0 = time.perf_counter()
        for _ in range(n_cold):
            engine.decode_step(True)
        sync_all()
        cold_ms = (time.perf_counter() - t0) * 1e3 / n_cold
        for _ in range(args.settle_steps - n_cold):
            engine.decode_step(True)
    start()
    for _ in range(args.warmup):
        engine.decode_step(True)
    sync_all()
    t0 = time.perf_counter()
    for _ in range(args.steps):
        engine.decode_step(True)
    sync_all()
    dt = time.perf_counter() - t0
    if dist is not None:
        # (a gloo group, the one-GPU rehearsal, is given host tensors only)
        t = torch.tensor([dt], device="cpu" if dist.get_backend() == "gloo" else dev, dtype=torch.float64)
        dist.all_reduce(t, op=dist.ReduceOp.MAX)
        dt = float(t.item())
    if hasattr(engine, "check_collectives"):
        engine.check_collectives()      # a timed-out device wait (one-shot or two-shot) must fail the run, not colour it
    timed_decode.cold_ms = cold_ms
    return dt


def main(argv=None):
    args = parse_args(argv)
    in_job = "WORLD_SIZE" in os.environ and "RANK" in os.environ
    if args.gpus > 1 and not in_job:
        # no torchrun environment: become the launcher (nothing below has touched a GPU)
        raise SystemExit(launch_ranks(args.gpus, sys.argv[1:] if argv is None else argv))
    if args.probe:
        return probe_main(args)
    if args.layered:
        return layered_main(args)

    import torch
    world = int(os.environ.get("WORLD_SIZE", "1"))
    rank = int(os.environ.get("RANK", "0"))
    local_rank = int(os.environ.get("LOCAL_RANK", "0"))
    dev = torch.device("cuda", 0 if args.rehearsal else local_rank)
    torch.cuda.set_device(dev)
    dist = None
    rccl_world = 1
    if world > 1:
        import torch.distributed as dist
        os.environ.setdefault("MASTER_ADDR", "127.0.0.1")
        if args.rehearsal:
            dist.init_process_group("gloo")
            ones = torch.ones(1)
        else:
            dist.init_process_group("nccl", device_id=dev)
            ones = torch.ones(1, device=dev)
        dist.all_reduce(ones)                      # the collective really spans `world` ranks
        rccl_world = int(ones.item())

    from eventgpt_amd.data import EventImageProcessor, event_frames, synthetic_events

    tp = args.parallelism == "tp" and world > 1
    # tensor-parallel ranks are shards of ONE model and must see identical inputs;
    # data-parallel ranks are independent replicas with their own streams
    data_seed = 0 if (tp or world == 1) else rank
    torch.manual_seed(1234 + data_seed)
    cfg, model, model_name = build_model(args, dev)

    # The serving engine is built right after the model, before anything else has allocated and freed
    # device memory: its packed weights and caches then sit in memory handed out early, and the decode
    # step measures 1 % faster than with an engine built after the vision runs (2.675 vs 2.70 ms per token
    # on one box, same kernels; neither dropping the allocator's cache before the build nor expandable
    # segments nor an eager vision tower changes that).
    engine = build_engine(args, model, dist, tp, args.batch)

    # ---- event prefill: raster -> CLIP preprocess -> ViT -> projector -> pool
    proc = EventImageProcessor(cfg.vision_config.image_size)
    ev = synthetic_events(seed=data_seed)
    frames = event_frames(ev, args.frames)
    tens = [proc(f, return_tensors="pt")["pixel_values"][0].to(dev, torch.bfloat16) for f in frames]
    with torch.no_grad():
        for _ in range(2):
            feats = model.encode_event_frames(tens)
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        n_vis = 5
        for _ in range(n_vis):
            feats = model.encode_event_frames(tens)
        torch.cuda.synchronize()
        vision_ms = (time.perf_counter() - t0) * 1e3 / n_vis
    n_event = feats.shape[0]
    n_text = max(args.prompt_len - n_event, 1)
    text_ids = torch.randint(3, 32000, (n_text,), device=dev)
    with torch.no_grad():
        text = model.model.embed_tokens(text_ids)
        embeds = torch.cat([text[:35], feats.to(text.dtype), text[35:]])  # splice position of <event>
    S = embeds.shape[0]

    # ---- LLM prefill latency (one stream; sharded over the TP group when there is one)
    def prefill_once():
        engine.reset()
        engine.prefill(embeds, select="greedy" if args.batch == 1 else None)

    for _ in range(2):
        prefill_once()
    torch.cuda.synchronize()
    n_pf = 5
    t0 = time.perf_counter()
    for _ in range(n_pf):
        prefill_once()
    torch.cuda.synchronize()
    prefill_ms = (time.perf_counter() - t0) * 1e3 / n_pf

    # ---- decode
    dt = timed_decode(args, engine, embeds, args.batch, dist, dev)
    cold_ms = timed_decode.cold_ms
    streams = (1 if tp else world) * args.batch
    tok_s = streams * args.steps / dt
    graph_captured = bool(engine.graph_captured)
    graph_fallback = engine.graph_fallback
    tp_allreduce = getattr(engine, "allreduce_kind", "none")

    extra = {}
    printed = threading.Lock()

    def line() -> dict:
        return {
            "metric": "decode tokens/sec (EventGPT-7B bf16 greedy, bs 1 per stream)" if args.batch == 1
            else f"decode tokens/sec (EventGPT-7B bf16 greedy, {args.batch} streams per engine)",
            "value": round(tok_s, 2), "unit": "tokens/s", "n_gpus": world, "steps": args.steps,
            "warmup": args.warmup, "settle_steps": args.settle_steps,
            "ms_per_step": round(dt * 1e3 / args.steps, 4),
            **({} if cold_ms is None else {"ms_per_step_cold": round(cold_ms, 4)}),
            "higher_is_better": True,
            "scaling": "strong" if (tp or world == 1) else "weak",
            "vs_baseline": round(tok_s / BASELINE_DECODE_TOK_S, 3),
            "dtype": "bf16" if args.weight_format == "bf16" else f"bf16 compute, {args.weight_format} weights",
            "data": "synthetic event stream, random-init weights",
            "event_prefill_ms": round(prefill_ms, 3),
            "event_prefill_vs_baseline": round(BASELINE_PREFILL_MS / prefill_ms, 3),
            "vision_ms_per_frame": round(vision_ms / args.frames, 3),
            "vision_vs_baseline": round(BASELINE_VISION_MS / (vision_ms / args.frames), 3),
            "rccl_world_size": rccl_world, **({"rehearsal_backend": "gloo"} if args.rehearsal else {}),
            "graph_captured": graph_captured,
            "graph_fallback": graph_fallback, "tp_allreduce": tp_allreduce,
            **dict(extra),
            "config": {"model": model_name, "global_batch": streams, "seq_len": S,
                       "event_frames": args.frames,
                       "parallelism": f"{args.parallelism}{world}"},
        }

    def emit() -> None:
        """Rank 0's one JSON line; whichever of the normal end and the extras' time limit comes first."""
        if rank != 0 or not printed.acquire(blocking=False):
            return
        print(json.dumps(line()), flush=True)

    # ---- extras (never the value).  They run after the headline measurement and must not be able
    # to cost it: an exception is reported under the extra's key (every rank takes the same
    # branch, so the group stays in step), and if the extras as a whole outlast their time limit
    # -- ranks waiting in a collective that one of them has left -- every rank prints what it
    # has, ends its child job and ends the process.
    multi = tp and args.batch == 1
    plan = []
    if multi and not args.no_batch32:
        plan.append("tp_batch32")
    if multi and not args.no_dp_extra:
        plan.append("dp_replicas")
    if multi and not args.no_dp_train_extra:
        plan.append("dp_train")
    if multi and not args.no_sd_extra:
        plan.append("sd_two_gpu")
    if multi and not args.no_oneshot_extra and tp_allreduce in ("rccl", "gloo"):
        plan.append("tp_oneshot")          # last: the one extra whose code has never run on this fabric
    if plan and args.extras_timeout > 0:
        def give_up():
            for name in plan:
                extra.setdefault(name, {"error": f"not finished within {args.extras_timeout} s"})
            kill_children()
            emit()
            sys.stdout.flush()
            os._exit(0)
        watchdog = threading.Timer(args.extras_timeout, give_up)
        watchdog.daemon = True
        watchdog.start()
    else:
        watchdog = None
    if args.extras_stall > 0:
        torch.cuda.synchronize()
        time.sleep(args.extras_stall)

    def free_headline_engine():
        nonlocal engine, model
        if engine is not None and hasattr(engine, "close"):
            engine.close()                 # peer mappings go in an order all ranks agree on
        engine = model = None
        torch.cuda.empty_cache()

    # the batched TP configuration (32 event streams), same group, same run
    if "tp_batch32" in plan:
        free_headline_engine()
        eng32 = model32 = None
        try:
            _, model32, _ = build_model(args, dev)
            eng32 = build_engine(args, model32, dist, True, 32)
            dt32 = timed_decode(args, eng32, embeds, 32, dist, dev)
            extra["tp_batch32"] = {"tokens_per_s": round(32 * args.steps / dt32, 2),
                                   "ms_per_step": round(dt32 * 1e3 / args.steps, 4), "global_batch": 32,
                                   "graph_captured": bool(eng32.graph_captured),
                                   "tp_allreduce": getattr(eng32, "allreduce_kind", "none")}
        except Exception as e:
            extra["tp_batch32"] = {"error": str(e)[:200]}
        try:
            if eng32 is not None:
                eng32.close()
        except Exception:
            pass
        eng32 = model32 = None
    # independent replicas on the same GPUs (no communication in the step): the fabric-free
    # bound the tensor-parallel numbers can be read against
    if "dp_replicas" in plan:
        free_headline_engine()
        try:
            _, model_dp, _ = build_model(args, dev)
            eng_dp = build_engine(args, model_dp, None, False, 1)
            dt_dp = timed_decode(args, eng_dp, embeds, 1, dist, dev)
            extra["dp_replicas"] = {"tokens_per_s": round(world * args.steps / dt_dp, 2),
                                    "ms_per_step": round(dt_dp * 1e3 / args.steps, 4), "global_batch": world,
                                    "scaling": "weak", "graph_captured": bool(eng_dp.graph_captured)}
        except Exception as e:
            extra["dp_replicas"] = {"error": str(e)[:200]}
        eng_dp = model_dp = None
    # one fine-tuning step per rank through the sharded AdamW's reduce-scatter / all-gather
    if "dp_train" in plan:
        free_headline_engine()
        try:
            from eventgpt_amd.benchmarks.multi_gpu_extras import dp_train_extra
            extra["dp_train"] = dp_train_extra(args.model, dist, dev, world, rank,
                                               steps=min(max(args.steps // 4, 2), 8), warmup=2)
        except Exception as e:
            extra["dp_train"] = {"error": f"{type(e).__name__}: {e}"[:200]}
        torch.cuda.empty_cache()
    # prefill hiding with the verifier on rank 1's GPU (rank 0 drives both devices, the others wait)
    if "sd_two_gpu" in plan:
        free_headline_engine()
        on_host = dist.get_backend() == "gloo"
        try:
            if rank == 0:
                from eventgpt_amd.benchmarks.multi_gpu_extras import sd_two_gpu_extra
                dev1 = dev if (args.rehearsal or torch.cuda.device_count() < 2) else torch.device("cuda", 1)
                short = args.model != "7b"
                extra["sd_two_gpu"] = sd_two_gpu_extra(args.model, dev, dev1, new_tokens=24 if short else 50,
                                                       drafter_prompt=120 if short else 636,
                                                       verifier_prompt=400 if short else 2115)
        except Exception as e:
            extra["sd_two_gpu"] = {"error": f"{type(e).__name__}: {e}"[:200]}
        torch.cuda.set_device(dev)
        torch.cuda.empty_cache()
        flag = torch.zeros(1, device="cpu" if on_host else dev)
        dist.all_reduce(flag)              # the others wait here for rank 0
    # the same tensor-parallel measurement on the in-tree all-reduce, as a child job of every rank
    # (8 ranks: 16 processes hold a GPU for its duration, two per device)
    if "tp_oneshot" in plan:
        free_headline_engine()
        if rank == 0:
            # whatever the child job does to this machine, the line as it stands is on record
            snap = json.dumps(line())
            print("[bench] line before the in-tree all-reduce child job: " + snap, file=sys.stderr, flush=True)
            try:
                os.makedirs("gpurun_out", exist_ok=True)
                with open(os.path.join("gpurun_out", "bench_line_before_oneshot.json"), "w") as f:
                    f.write(snap + "\n")
            except OSError:
                pass
        try:
            got = run_oneshot_child(args, dist, rank, world, local_rank, dev)
            if got is not None:
                extra["tp_oneshot"] = got
        except Exception as e:
            extra["tp_oneshot"] = {"error": f"{type(e).__name__}: {e}"[:200]}
    if watchdog is not None:
        watchdog.cancel()
    emit()
    if engine is not None and hasattr(engine, "close"):
        try:
            engine.close()
        except Exception:
            pass
    if dist is not None:
        dist.destroy_process_group()


if __name__ == "__main__":
    main()
