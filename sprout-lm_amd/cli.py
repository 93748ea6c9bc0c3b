"""Command line of the engine.

    python -m sprout_lm_amd demo [--json] [--pressure]
    python -m sprout_lm_amd generate MODEL_DIR --prompt-ids 1,2,3 [--max-new-tokens N] ...
    python -m sprout_lm_amd init --preset tiny-a|tiny-b|qwen2.5-0.5b|megozen-s|bogilix-s|morarax-s|kodezen-s|lozupel-s|varunex-s|... | --config FILE  --out DIR [--seed N]

`demo` is the counterpart of the reference's src/demo.ts, with the reference's two options: a few requests on a
tiny random model, told round by round (--json: the same as one JSON document; --pressure: a pool so small that
requests are preempted and their cache is computed again).  `generate` follows
scripts/smoke-cuda.ts: one prompt on a model folder, one JSON line per scheduling round and a final
report; the reference's environment variables MAX_NEW_TOKENS, KV_TOKENS, MAX_SEQUENCES,
PREFILL_CHUNK_SIZE and REPORT_PATH are honoured as defaults of the options of the same meaning.
There is no tokenizer: prompts are token ids.
"""
from __future__ import annotations

import argparse
import json
import os
import sys
import tempfile
import time

PRESETS = {
    "tiny-a": dict(model_type="qwen2", hidden_act="silu", hidden_size=64, intermediate_size=128, num_hidden_layers=2,
                   num_attention_heads=4, num_key_value_heads=2, vocab_size=256, max_position_embeddings=128,
                   rms_norm_eps=1e-6, rope_theta=10000.0, tie_word_embeddings=True, eos_token_id=255),
    "tiny-b": dict(model_type="qwen2", hidden_act="silu", hidden_size=96, intermediate_size=224, num_hidden_layers=3,
                   num_attention_heads=3, num_key_value_heads=1, vocab_size=384, max_position_embeddings=256,
                   rms_norm_eps=1e-5, rope_theta=1000000.0, tie_word_embeddings=False, eos_token_id=383),
    "qwen2.5-0.5b": dict(model_type="qwen2", hidden_act="silu", hidden_size=896, intermediate_size=4864,
                         num_hidden_layers=24, num_attention_heads=14, num_key_value_heads=2, vocab_size=151936,
                         max_position_embeddings=32768, rms_norm_eps=1e-6, rope_theta=1000000.0,
                         tie_word_embeddings=True, eos_token_id=151643),
    "qwen2.5-7b": dict(model_type="qwen2", hidden_act="silu", hidden_size=3584, intermediate_size=18944,
                       num_hidden_layers=28, num_attention_heads=28, num_key_value_heads=4, vocab_size=152064,
                       max_position_embeddings=32768, rms_norm_eps=1e-6, rope_theta=1000000.0,
                       tie_word_embeddings=False, eos_token_id=151643),
    "qwen2.5-32b": dict(model_type="qwen2", hidden_act="silu", hidden_size=5120, intermediate_size=27648,
                        num_hidden_layers=64, num_attention_heads=40, num_key_value_heads=8, vocab_size=152064,
                        max_position_embeddings=32768, rms_norm_eps=1e-6, rope_theta=1000000.0,
                        tie_word_embeddings=False, eos_token_id=151643),
}


def _megozen_preset(width: int, layers: int, heads: int, dim: int, rot_dim: int, vdim: int, kv_rank: int, experts: int,
                    top: int, ff: int, shared_ff: int, window: int | None, vocab: int, own: int | None = None) -> dict:
    """A Megozen configuration of `layers` equal layers, of which the first `own` have tensors (the others run with
    those of layer i mod own)."""
    mixer = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank,
             "scale": (dim + rot_dim) ** -0.5,
             "rot": {"base": 500000.0, "dims": rot_dim, "scaling": {"factor": 4.0, "original": 4096, "fast": 32.0, "slow": 1.0}}}
    if window:
        mixer["mask"] = {"size": window}
    mlp = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}, "shared": {"ff": shared_ff}}
    own = own or layers
    entries = [dict({"type": "latent_attention", "mixer": mixer, "mlp": mlp}, **({"weights_of": i % own} if i >= own else {}))
               for i in range(layers)]
    return {"architecture": "Megozen", "vocab": vocab, "width": width, "norm": {"eps": 1e-6},
            "embedding": {"bigram": {"buckets": 65521, "mul_prev": 8191, "mul_cur": 131}}, "layers": entries}


def _dense_twin(width: int, layers: int, heads: int, kv_heads: int, inner: int, vocab: int) -> dict:
    """The dense Qwen2 layer sizes that compute as much per token as a Megozen preset: the same width, layers and
    vocabulary, `inner` = what a token's chosen experts and the shared one hold together."""
    return dict(model_type="qwen2", hidden_act="silu", hidden_size=width, intermediate_size=inner, num_hidden_layers=layers,
                num_attention_heads=heads, num_key_value_heads=kv_heads, vocab_size=vocab, max_position_embeddings=32768,
                rms_norm_eps=1e-6, rope_theta=1000000.0, tie_word_embeddings=False, eos_token_id=0)


PRESETS.update({
    # small: 8 layers of width 1,024 (4 with tensors, each run twice), a window of 1,024 keys
    "megozen-s": _megozen_preset(1024, 8, 8, 64, 32, 64, 96, 16, 2, 512, 1024, 1024, 32768, own=4),
    "megozen-s-dense": _dense_twin(1024, 8, 8, 1, 2048, 32768),
    # medium: 12 layers of width 2,048, every earlier key visible
    "megozen-m": _megozen_preset(2048, 12, 16, 64, 32, 64, 96, 32, 4, 704, 1408, None, 32768),
    "megozen-m-dense": _dense_twin(2048, 12, 16, 2, 4224, 32768),
    # large: 8 layers of width 4,096, 32 heads over one latent
    "megozen-l": _megozen_preset(4096, 8, 32, 64, 32, 64, 96, 64, 6, 1024, 2048, None, 32768),
    "megozen-l-dense": _dense_twin(4096, 8, 32, 4, 8192, 32768),
})


def _bogilix_preset(width: int, layers: int, heads: int, kv_heads: int, dim: int, normed_dim: int, chunk: int, experts: int,
                    identity: int, top: int, ff: int, shared_ff: int, dense_ff: int, vocab: int) -> dict:
    """A Bogilix configuration: three layers with normed queries and keys (heads of `normed_dim`, capped scores) to one
    with rotated ones (heads of `dim`), values of `dim`, blocks of `chunk` positions (twice that in the rotated layers);
    the first layer's feed-forward dense, the others routed (four groups of which two stay open)."""
    def mixer(kind):
        m = {"heads": heads, "kv_heads": kv_heads, "vdim": dim, "v_mix": True}
        if kind == "attention":
            m.update({"dim": dim, "scale": dim ** -0.5, "mask": {"size": 2 * chunk}, "rot": {"base": 500000.0, "dims": dim}})
        else:
            m.update({"dim": normed_dim, "scale": normed_dim ** -0.5, "mask": {"size": chunk}, "softcap": 30.0})
        return m
    moe = {"kind": "moe", "expert": {"ff": ff, "limit": 7.0}, "shared": {"ff": shared_ff, "limit": 7.0},
           "router": {"experts": experts, "identity": identity, "top": top, "scale": 2.5, "groups": {"count": 4, "keep": 2}}}
    entries = []
    for i in range(layers):
        kind = "attention" if i % 4 == 3 else "attention_2"
        entries.append({"type": kind, "mixer": mixer(kind), "mlp": {"kind": "dense", "ff": dense_ff} if i == 0 else moe})
    return {"architecture": "Bogilix", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "layers": entries}


PRESETS.update({
    # small: 8 layers of width 1,024, 16 heads of 64 over 2 key/value heads, blocks of 1,024 and 2,048 positions
    "bogilix-s": _bogilix_preset(1024, 8, 16, 2, 64, 48, 1024, 14, 2, 2, 512, 1024, 2048, 32768),
    "bogilix-s-dense": _dense_twin(1024, 8, 16, 2, 2048, 32768),
    # medium: 12 layers of width 2,048, 16 heads of 128 (normed layers: keys of 96 beside values of 128)
    "bogilix-m": _bogilix_preset(2048, 12, 16, 2, 128, 96, 1024, 30, 2, 4, 704, 1408, 4224, 32768),
    "bogilix-m-dense": _dense_twin(2048, 12, 16, 2, 4224, 32768),
    # large: 8 layers of width 4,096, 32 heads of 128 over 4 key/value heads
    "bogilix-l": _bogilix_preset(4096, 8, 32, 4, 128, 128, 2048, 62, 2, 6, 1024, 2048, 8192, 32768),
    "bogilix-l-dense": _dense_twin(4096, 8, 32, 4, 8192, 32768),
})


def _morarax_preset(width: int, layers: int, heads: int, kv_heads: int, dim: int, state_heads: int, blocks: int, ff: int,
                    vocab: int) -> dict:
    """A Morarax configuration: layers in the order retention, gated recurrence, retention, attention, again and again.
    Attention heads of `dim` with blended frequencies; retention heads of 64 keys beside 128 values with decays
    1 - 2^(-5 - 4 h / heads); a recurrence as wide as the model in `blocks` parts behind four taps."""
    attention = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5,
                 "rot": {"base": 500000.0, "dims": dim // 2, "scaling": {"factor": 4.0, "original": 4096, "fast": 32.0, "slow": 1.0}}}
    retention = {"heads": state_heads, "dim": 64, "vdim": 128, "rot": {"base": 10000.0, "dims": 64},
                 "decay": [1.0 - 2.0 ** (-5.0 - 4.0 * h / state_heads) for h in range(state_heads)]}
    recurrence = {"width": width, "blocks": blocks, "conv": 4}
    order = (("retention", retention), ("rglru", recurrence), ("retention", retention), ("attention", attention))
    entries = [{"type": order[i % 4][0], "mixer": order[i % 4][1], "mlp": {"kind": "dense", "ff": ff}} for i in range(layers)]
    return {"architecture": "Morarax", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "residual_mult": 0.5,
            "logit_scale": 0.25, "layers": entries}


PRESETS.update({
    # small: 8 layers of width 1,024; attention of 16 heads of 64 over 2 key/value heads, retention of 8 heads
    "morarax-s": _morarax_preset(1024, 8, 16, 2, 64, 8, 16, 2048, 32768),
    "morarax-s-dense": _dense_twin(1024, 8, 16, 2, 2048, 32768),
    # medium: 12 layers of width 2,048; attention of 16 heads of 128, retention of 16 heads
    "morarax-m": _morarax_preset(2048, 12, 16, 2, 128, 16, 16, 4224, 32768),
    "morarax-m-dense": _dense_twin(2048, 12, 16, 2, 4224, 32768),
    # large: 8 layers of width 4,096; attention of 32 heads of 128 over 4 key/value heads, retention of 32 heads
    "morarax-l": _morarax_preset(4096, 8, 32, 4, 128, 32, 16, 8192, 32768),
    "morarax-l-dense": _dense_twin(4096, 8, 32, 4, 8192, 32768),
})


def _kodezen_preset(width: int, layers: int, heads: int, kv_heads: int, dim: int, ff: int, vocab: int) -> dict:
    """A Kodezen configuration: layers in the order mamba2, attention, mamba2, mamba1, again and again.  The state-space
    mixers are twice as wide as the model (mamba2: heads of 64 values, a state of 128 rows, two groups; mamba1: a state of
    16); attention heads of `dim` of which half turn, a window of 1,024 keys that keeps the first four.  Feed-forwards take
    turns: dense with `ff` * 3 / 2 inner numbers (two matrices where a gated one has three), and two of eight experts of
    `ff` / 2."""
    mamba2 = {"heads": 2 * width // 64, "vdim": 64, "state": 128, "groups": 2, "conv": 4, "norm_groups": 2}
    mamba1 = {"inner": 2 * width, "state": 16, "dt_rank": width // 16, "conv": 4}
    attention = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "conv": 3,
                 "rot": {"base": 500000.0, "dims": dim // 2}, "mask": {"size": 1024, "keep_first": 4}}
    order = (("mamba2", mamba2), ("attention", attention), ("mamba2", mamba2), ("mamba1", mamba1))
    dense = {"kind": "dense", "ff": ff * 3 // 2}
    moe = {"kind": "moe", "expert": {"ff": ff // 2}, "router": {"experts": 8, "top": 2}}
    entries = [{"type": order[i % 4][0], "mixer": order[i % 4][1], "mlp": moe if i % 2 else dense} for i in range(layers)]
    return {"architecture": "Kodezen", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "embedding": {"scale": width ** 0.5},
            "canon": {"taps": 4}, "layers": entries}


PRESETS.update({
    # beside each the closest design the engine has at equal width, layers, attention heads and feed-forward work: Morarax
    "kodezen-s": _kodezen_preset(1024, 8, 16, 2, 64, 2048, 32768),
    "kodezen-s-twin": _morarax_preset(1024, 8, 16, 2, 64, 8, 16, 2048, 32768),
    "kodezen-m": _kodezen_preset(2048, 12, 16, 2, 128, 4224, 32768),
    "kodezen-m-twin": _morarax_preset(2048, 12, 16, 2, 128, 16, 16, 4224, 32768),
    "kodezen-l": _kodezen_preset(4096, 8, 32, 4, 128, 8192, 32768),
    "kodezen-l-twin": _morarax_preset(4096, 8, 32, 4, 128, 32, 16, 8192, 32768),
})


def _lozupel_preset(width: int, layers: int, loop: tuple, heads: int, kv_heads: int, dim: int, delta_heads: int, delta_dim: int,
                    ff: int, vocab: int) -> dict:
    """A Lozupel configuration: layers in the order parallel, delta, again and again, layers loop[0] .. loop[1] - 1 run
    loop[2] times.  Sigmoid attention heads of `dim` in a window of 1,024 keys; delta-rule heads of `delta_dim` keys and
    values (in the delta layers two heads share a key head), convolutions of four taps, projections of decays and gates
    through `delta_dim` numbers."""
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "mask": {"size": 1024},
            "rot": {"base": 500000.0, "dims": dim}}
    right = {"heads": delta_heads, "kv_heads": delta_heads, "dim": delta_dim, "vdim": delta_dim, "conv": 4,
             "decay_rank": delta_dim, "gate_rank": delta_dim}
    delta = {"heads": delta_heads, "kv_heads": delta_heads // 2, "dim": delta_dim, "vdim": delta_dim, "conv": 4}
    order = (("parallel", {"left": left, "right": right}), ("delta", delta))
    entries = [{"type": order[i % 2][0], "mixer": order[i % 2][1], "mlp": {"kind": "dense", "ff": ff}} for i in range(layers)]
    return {"architecture": "Lozupel", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "embedding": {"scale": 3.0},
            "logit_softcap": 30.0, "loop": {"start": loop[0], "stop": loop[1], "times": loop[2]}, "layers": entries}


PRESETS.update({
    # beside each the closest design the engine has at equal width, layer runs, attention heads and feed-forward: Morarax
    # small: 6 layers of width 1,024, two of them run twice (8 runs)
    "lozupel-s": _lozupel_preset(1024, 6, (2, 4, 2), 16, 2, 64, 8, 128, 2048, 32768),
    "lozupel-s-twin": _morarax_preset(1024, 8, 16, 2, 64, 8, 16, 2048, 32768),
    # medium: 8 layers of width 2,048, two of them run three times (12 runs)
    "lozupel-m": _lozupel_preset(2048, 8, (2, 4, 3), 16, 2, 128, 16, 128, 4224, 32768),
    "lozupel-m-twin": _morarax_preset(2048, 12, 16, 2, 128, 16, 16, 4224, 32768),
    # large: 6 layers of width 4,096, two of them run twice (8 runs)
    "lozupel-l": _lozupel_preset(4096, 6, (2, 4, 2), 32, 4, 128, 32, 128, 8192, 32768),
    "lozupel-l-twin": _morarax_preset(4096, 8, 32, 4, 128, 32, 16, 8192, 32768),
})


def _varunex_preset(width: int, layers: int, heads: int, kv_heads: int, dim: int, latent: tuple, memory: tuple, ff: int, vocab: int) -> dict:
    """A Varunex configuration: layers in the order latent attention, memory, differential attention, memory, again and again.
    latent: heads, their unrotated and rotated numbers, the query and the key/value latents' sizes; memory: heads, key and value
    numbers; differential attention: `heads` heads of two maps of `dim` numbers over values of 2 dim in a window of 1,024 keys.
    Feed-forwards of ff * 3 / 2 inner numbers: two matrices where a gated one has three."""
    lat_heads, lat_dim, rot_dim, q_rank, kv_rank = latent
    attention = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": 2 * dim, "scale": dim ** -0.5, "diff": 0.5,
                 "mask": {"size": 1024}, "rot": {"base": 500000.0, "dims": dim,
                                                 "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}}
    latents = {"heads": lat_heads, "dim": lat_dim, "rot_dim": rot_dim, "vdim": lat_dim, "q_rank": q_rank, "kv_rank": kv_rank,
               "scale": (lat_dim + rot_dim) ** -0.5, "rot": {"base": 10000.0, "dims": rot_dim}}
    cells = {"heads": memory[0], "dim": memory[1], "vdim": memory[2], "gate_cap": 15.0}
    order = (("latent_attention", latents), ("mlstm", cells), ("attention", attention), ("mlstm", cells))
    entries = [{"type": order[i % 4][0], "mixer": order[i % 4][1], "mlp": {"kind": "dense", "ff": ff * 3 // 2}} for i in range(layers)]
    return {"architecture": "Varunex", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "layers": entries}


PRESETS.update({
    # beside each the closest design the engine has at equal width, layers, attention heads and feed-forward work: Morarax
    # small: keys of 96 + 32 beside each other, memories of 4 heads of 128 x 256
    "varunex-s": _varunex_preset(1024, 8, 16, 2, 32, (16, 64, 32, 384, 96), (4, 128, 256), 2048, 32768),
    "varunex-s-twin": _morarax_preset(1024, 8, 16, 2, 64, 8, 16, 2048, 32768),
    # medium: latents of 128 + 64, memories of 8 heads of 128 x 256
    "varunex-m": _varunex_preset(2048, 12, 16, 2, 64, (16, 128, 64, 768, 128), (8, 128, 256), 4224, 32768),
    "varunex-m-twin": _morarax_preset(2048, 12, 16, 2, 128, 16, 16, 4224, 32768),
    # large: latents of 128 + 64, memories of 8 heads of 256 x 512
    "varunex-l": _varunex_preset(4096, 8, 32, 4, 64, (32, 128, 64, 1536, 128), (8, 256, 512), 8192, 32768),
    "varunex-l-twin": _morarax_preset(4096, 8, 32, 4, 128, 32, 16, 8192, 32768),
})


def _env_int(name: str, default: int) -> int:
    value = os.environ.get(name)
    return default if value is None else int(value)


def preset_config(name: str):
    from .registry import config_from_dict
    return config_from_dict(PRESETS[name])


def cmd_init(args) -> int:
    import torch
    from .registry import config_from_dict
    from .weights.random_init import write_model_folder
    if args.config:
        with open(args.config) as f:
            config = config_from_dict(json.load(f))
    else:
        config = preset_config(args.preset)
    dtype = {"bfloat16": torch.bfloat16, "float32": torch.float32}[args.dtype]
    write_model_folder(args.out, config, args.seed, dtype=dtype, std=args.std)
    print(json.dumps({"written": args.out, "architecture": config.architecture, "seed": args.seed, "dtype": args.dtype}))
    return 0


def cmd_generate(args) -> int:
    from .runtime import create_runtime
    started = time.perf_counter()
    if args.prompt_ids:
        prompt = [int(t) for t in args.prompt_ids.split(",") if t.strip()]
    else:
        import random
        rng = random.Random(args.seed)
        prompt = None
    runtime = create_runtime(args.model, args.dtype, max_context_tokens=args.kv_tokens, block_size=args.block_size,
                             max_sequences=args.max_sequences, max_batch_tokens=args.max_batch_tokens,
                             prefill_chunk_size=args.prefill_chunk_size, prefix_caching=not args.no_prefix_caching,
                             step_token_multiple=args.step_token_multiple, weight_limit_mib=args.weight_limit_mib,
                             reserve_mib=args.reserve_mib, strict_tensors=args.strict_tensors)
    engine = runtime.engine
    if prompt is None:
        prompt = [rng.randrange(engine.model.vocab_size) for _ in range(args.prompt_len)]
    load_ms = (time.perf_counter() - started) * 1000
    print(json.dumps({"phase": "ready", "name": runtime.name, "input": prompt, "load_ms": round(load_ms, 1),
                      "notes": getattr(engine.model, "load_notes", [])}), flush=True)
    engine.add("cli", prompt, args.max_new_tokens, temperature=args.temperature, seed=args.seed,
               ignore_eos=args.ignore_eos)
    rounds, first_token_ms = [], None
    generation = time.perf_counter()
    while engine.pending:
        before = time.perf_counter()
        report = engine.step()
        tokens = [e["token"] for e in report.events if e["type"] == "token"]
        if tokens and first_token_ms is None:
            first_token_ms = (time.perf_counter() - generation) * 1000
        record = {"round": len(rounds) + 1, "ms": round((time.perf_counter() - before) * 1000, 3),
                  "phase": report.work[0]["phase"] if report.work else "none", "tokens": tokens}
        rounds.append(record)
        if not args.quiet:
            print(json.dumps(record), flush=True)
    generation_ms = (time.perf_counter() - generation) * 1000
    result = engine.result("cli")
    decode = [r for r in rounds if r["phase"] == "decode"]
    decode_ms = sum(r["ms"] for r in decode)
    report = {"model": runtime.name, "input": prompt, "output": result["output"], "finish_reason": result["finish_reason"],
              "load_ms": load_ms, "first_token_ms": first_token_ms, "generation_ms": generation_ms,
              "decode_summary": {"steps": len(decode), "total_ms": decode_ms,
                                 "mean_ms": decode_ms / len(decode) if decode else None,
                                 "steps_per_second": len(decode) * 1000 / decode_ms if decode_ms else None},
              "stats": runtime.stats(), "rounds": rounds}
    if args.report:
        os.makedirs(os.path.dirname(os.path.abspath(args.report)), exist_ok=True)
        with open(args.report, "w") as f:
            json.dump(report, f, indent=2)
    print(json.dumps({"phase": "finished", "output": result["output"], "finish_reason": result["finish_reason"],
                      "first_token_ms": first_token_ms, "generation_ms": generation_ms,
                      "decode_summary": report["decode_summary"]}))
    runtime.close()
    return 0


def cmd_demo(args) -> int:
    """A few rounds of the engine on a tiny random model, told round by round.

    Four requests with random token ids: `long` (a prompt that needs several portions), `short`, `twin` (it
    starts with the first 16 tokens of `long` and arrives a round later, so it finds two of its pages in the
    cache) and `late`, which arrives while the others decode and samples with a temperature.  Every round prints the one batch that the
    model ran: portions of prompts beside single decoded tokens, flat in one step; whether the step was replayed
    from a recorded graph and in which bucket (sequences, context); whether the round after it was already on the
    GPU when this one's tokens came back; and what the cache pool looks like.  --pressure makes the pool so small
    that requests lose their pages to older ones and compute them again.
    """
    import random

    import torch
    from .engine.engine import Engine
    from .weights.random_init import write_model_folder
    config = preset_config("tiny-b")
    page, pages = 8, (9 if args.pressure else 24)
    with tempfile.TemporaryDirectory() as folder:
        write_model_folder(folder, config, seed=2, dtype=torch.bfloat16, std=0.08)
        engine = Engine.from_folder(folder, args.dtype, block_size=page, num_blocks=pages, max_sequences=3,
                                    max_batch_tokens=24, prefill_chunk_size=16, record_trace=True)
    rng = random.Random(5)
    ids = lambda n: [rng.randrange(config.vocab_size - 2) for _ in range(n)]
    long_prompt = ids(40)
    # before which round each request arrives: `twin` after `long` has computed (and offered) its first pages
    arrivals = {0: [("long", long_prompt, 10, {}), ("short", ids(6), 12, {})],
                1: [("twin", long_prompt[:16] + ids(5), 8, {})],
                5: [("late", ids(11), 6, {"temperature": 0.8, "seed": 7})]}
    say = (lambda *a: None) if args.json else print
    say(f"sprout-lm_amd demo: {config.num_hidden_layers}-layer Qwen2 of random weights in {args.dtype} on "
        f"{torch.cuda.get_device_name()}; {pages} pages of {page} tokens, 3 sequences, 24 tokens a step")
    say("(token ids only: the weights are untrained, what is shown is the engine at work)\n")
    from .engine.graphs import _bucket
    rounds, round_no = [], 0
    while engine.pending or any(r >= round_no for r in arrivals):
        for name, prompt, new, sampling in arrivals.get(round_no, []):
            engine.add(name, prompt, new, ignore_eos=True, **sampling)
        round_no += 1
        if round_no > 500:
            raise RuntimeError("the demo's requests did not finish in 500 rounds")
        report = engine.step()
        graphs = engine.model._graphs
        replayed = report.replayed
        bucket = None
        if replayed:     # the recorded graph of this many sequences (rounded up to a power of two), last used first
            bucket = next((k for k in reversed(list(graphs.graphs)) if k[0] == _bucket(len(report.work))), None)
        record = {"round": round_no, "work": report.work, "events": report.events, "from_graph": replayed,
                  "graph_bucket": bucket, "launched_ahead": report.launched_ahead,
                  "next_round_already_launched": engine._ahead is not None,
                  "free_pages": report.memory["free_pages"], "cached_pages": report.memory["cached_pages"]}
        rounds.append(record)
        if args.json:
            continue
        batch = " + ".join(f"{w['tokens']} of {w['id']} ({w['phase']} from {w['from']})" for w in report.work) or "nothing to run"
        how = "launched kernel by kernel"
        if replayed:
            how = f"graph replay, bucket {bucket[0]} sequences x {bucket[1]} keys" if bucket else "graph replay"
            how += " (launched during the round before)" if report.launched_ahead else ""
        ahead = "; the next round is already on the GPU" if record["next_round_already_launched"] else ""
        say(f"round {round_no:>2}: one batch of {sum(w['tokens'] for w in report.work)} tokens = {batch}")
        say(f"          {how}{ahead}; pages free {record['free_pages']}/{pages}, kept for reuse {record['cached_pages']}")
        for event in report.events:
            if event["type"] != "token":
                say(f"          {event['id']}: {event['type']} - {event['detail']}")
        made = {e['id']: e['token'] for e in report.events if e['type'] == 'token'}
        if made:
            say("          new tokens: " + ", ".join(f"{k} -> {v}" for k, v in made.items()))
    results = {name: engine.result(name) for name in ("long", "short", "twin", "late")}
    stats = engine.stats()
    replays = engine.model._graphs.replays if engine.model._graphs else 0
    summary = {"mode": "pressure" if args.pressure else "roomy", "rounds": rounds, "results": results, "stats": stats,
               "graphs_recorded": len(engine.model._graphs.graphs) if engine.model._graphs else 0, "graph_replays": replays}
    if args.json:
        print(json.dumps(summary, indent=2))
    else:
        say("\nwhat came out:")
        for name, r in results.items():
            say(f"  {name:>5}: {r['status']} ({r['finish_reason']}), {r['prefix_hits']} prompt tokens found in the cache, "
                f"preempted {r['preemptions']} times, output {r['output']}")
        say(f"  {stats['preemptions']} preemptions, {stats['recomputed_tokens']} tokens computed again, "
            f"{summary['graphs_recorded']} graphs recorded and replayed {replays} times in {round_no} rounds")
    engine.close()
    return 0


def main(argv=None) -> int:
    parser = argparse.ArgumentParser(prog="python -m sprout_lm_amd", description=__doc__,
                                     formatter_class=argparse.RawDescriptionHelpFormatter)
    sub = parser.add_subparsers(dest="command", required=True)

    demo = sub.add_parser("demo", help="four requests on a tiny random model, round by round")
    demo.add_argument("--json", action="store_true")
    demo.add_argument("--pressure", action="store_true", help="a pool of 9 pages: requests are preempted")
    demo.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    demo.set_defaults(run=cmd_demo)

    gen = sub.add_parser("generate", help="one prompt of token ids on a model folder")
    gen.add_argument("model", nargs="?", default=os.environ.get("MODEL_DIR"))
    gen.add_argument("--prompt-ids", help="comma-separated token ids")
    gen.add_argument("--prompt-len", type=int, default=16, help="random prompt of this length if no --prompt-ids")
    gen.add_argument("--max-new-tokens", type=int, default=_env_int("MAX_NEW_TOKENS", 4))
    gen.add_argument("--temperature", type=float, default=0.0)
    gen.add_argument("--seed", type=int, default=0)
    gen.add_argument("--ignore-eos", action="store_true")
    gen.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    gen.add_argument("--kv-tokens", type=int, default=_env_int("KV_TOKENS", 2048))
    gen.add_argument("--block-size", type=int, default=16)
    gen.add_argument("--max-sequences", type=int, default=_env_int("MAX_SEQUENCES", 4))
    gen.add_argument("--max-batch-tokens", type=int, default=2048)
    gen.add_argument("--prefill-chunk-size", type=int, default=_env_int("PREFILL_CHUNK_SIZE", 512))
    gen.add_argument("--step-token-multiple", type=int, default=1,
                     help="cut a step of more tokens than this back to a whole multiple of it (1: off)")
    gen.add_argument("--no-prefix-caching", action="store_true")
    gen.add_argument("--weight-limit-mib", type=int, default=_env_int("CUDA_WEIGHT_LIMIT_MIB", 0),
                     help="most device memory the weights may take (0: no limit)")
    gen.add_argument("--reserve-mib", type=int, default=_env_int("CUDA_RESERVE_MIB", 1024),
                     help="device memory that must stay free after weights and cache pools")
    gen.add_argument("--strict-tensors", action="store_true",
                     help="refuse a checkpoint that holds tensors the model does not ask for")
    gen.add_argument("--report", default=os.environ.get("REPORT_PATH"), help="write the full JSON report here")
    gen.add_argument("--quiet", action="store_true")
    gen.set_defaults(run=cmd_generate)

    init = sub.add_parser("init", help="write a model folder with seeded random weights")
    init.add_argument("--preset", choices=sorted(PRESETS))
    init.add_argument("--config", help="a config.json to take sizes from")
    init.add_argument("--out", required=True)
    init.add_argument("--seed", type=int, default=0)
    init.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    init.add_argument("--std", type=float, default=0.02)
    init.set_defaults(run=cmd_init)

    args = parser.parse_args(argv)
    if args.command == "generate" and not args.model:
        parser.error("generate needs a model folder (argument or MODEL_DIR)")
    if args.command == "init" and not (args.preset or args.config):
        parser.error("init needs --preset or --config")
    return args.run(args)
