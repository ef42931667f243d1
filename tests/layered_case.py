"""Helpers of the tests of decoders of listed layers: model folders, schedules played through the framework's trace replay,
engines and greedy generation."""
import json
import os

import torch


def write_model(folder, cfg, weights):
    """A model folder; the safetensors file is written here, byte by byte as the format says."""
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    header, blobs, at = {}, [], 0
    for name, t in weights.items():
        raw = t.bfloat16().contiguous().view(torch.int16).numpy().tobytes()
        header[name] = {"dtype": "BF16", "shape": list(t.shape), "data_offsets": [at, at + len(raw)]}
        blobs.append(raw)
        at += len(raw)
    head = json.dumps(header).encode()
    with open(os.path.join(folder, "model.safetensors"), "wb") as f:
        f.write(len(head).to_bytes(8, "little") + head + b"".join(blobs))
    return str(folder)


def tokens(cfg, n, seed):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(1000 + seed)).tolist()


def error(got, want):
    """RMS over the vocabulary of the difference (means taken off) per row, in units of the expected logits' spread."""
    d = got.double() - want
    d = d - d.mean(1, keepdim=True)
    return d.pow(2).mean(1).sqrt() / want.std()


def replay(folder, dtype, max_tokens):
    from light_vllm_amd.engine.registry import load_model_config
    from light_vllm_amd.engine.trace import TraceReplay
    return TraceReplay(load_model_config(folder, dtype), max_tokens)


def play(rp, requests, steps):
    """requests {id: tokens}; steps [[(id, n), ...], ...] -> {id: logits of all its tokens}.  A request ends with its last
    token."""
    at, out = {}, {rid: [] for rid in requests}
    for step in steps:
        entries = []
        for rid, n in step:
            a = at.get(rid, 0)
            entries.append((rid, requests[rid][a:a + n], list(range(n))))
            at[rid] = a + n
        logits = rp.step(entries)
        row = 0
        for rid, n in step:
            out[rid].append(logits[row:row + n])
            row += n
            if at[rid] == len(requests[rid]):
                rp.end(rid)
    return {rid: torch.cat(o) for rid, o in out.items()}


def portions(n, sizes):
    """n cut into portions of the given sizes in turn."""
    out, i = [], 0
    while n > 0:
        k = min(n, sizes[i % len(sizes)])
        out.append(k)
        n, i = n - k, i + 1
    return out


def engine(folder, dtype, graph=True, num_blocks=64, max_seqs=8, chunked=False, budget=512, cache=None, **kw):
    from light_vllm_amd.engine.config import CacheConfig, SchedulerConfig
    from light_vllm_amd.engine.llm_engine import LLMEngine
    return LLMEngine.from_pretrained(
        folder, dtype, CacheConfig(num_gpu_blocks=num_blocks, num_cpu_blocks=32, **(cache or {})),
        SchedulerConfig(max_num_batched_tokens=budget, max_num_seqs=max_seqs, max_model_len=256,
                        chunked_prefill_enabled=chunked, **kw), use_hip_graph=graph)


def generate(eng, prompts, n, use_async=False):
    for i, p in enumerate(prompts):
        eng.add_request(str(i), p, max_tokens=n)
    done = {}
    step = eng.async_step if use_async else eng.step
    for _ in range(2000):
        for out in step():
            if out.finished:
                done[int(out.request_id)] = out.token_ids
        if not eng.has_unfinished_requests() and eng.num_on_the_fly == 0:
            break
    eng.shutdown()
    return [done[i] for i in range(len(prompts))]


def greedy(forward, prompt, n):
    """forward(tokens) -> logits: the arg-max continuation."""
    t = list(prompt)
    for _ in range(n):
        t.append(int(forward(t)[-1].argmax()))
    return t[len(prompt):]
