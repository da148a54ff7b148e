"""``automodel`` CLI: YAML in, recipe out.

Reference behavior: nemo_automodel/cli/app.py:95-159 (parse YAML, resolve the
``recipe:`` target, dispatch to a launcher). Usage:

    automodel <cfg.yaml> [--nproc-per-node N] [--a.b.c=v ...]
    automodel capabilities [ARCHITECTURE]
    automodel generate --model DIR --prompt-ids 5,17,3 [--prompt-ids ...]
"""

from __future__ import annotations

import sys

from automodel_amd.config.loader import (
    apply_overrides,
    load_yaml_config,
    parse_cli_overrides,
    resolve_target,
)

RECIPE_ALIASES = {
    "llm_finetune": "automodel_amd.recipes.llm.train_ft.TrainFinetuneRecipeForNextTokenPrediction",
    "llm_pretrain": "automodel_amd.recipes.llm.train_ft.TrainFinetuneRecipeForNextTokenPrediction",
    "llm_benchmark": "automodel_amd.recipes.llm.benchmark.BenchmarkingRecipeForNextTokenPrediction",
    "vlm_finetune": "automodel_amd.recipes.vlm.finetune.FinetuneRecipeForVLM",
    "llm_kd": "automodel_amd.recipes.llm.kd.KDRecipeForNextTokenPrediction",
    "llm_seq_cls": "automodel_amd.recipes.llm.train_seq_cls.TrainFinetuneRecipeForSequenceClassification",
    "retrieval": "automodel_amd.recipes.llm.train_retrieval.TrainRecipeForRetrieval",
    "eagle_draft": "automodel_amd.speculative.train_draft.TrainEagleDraftRecipe",
    "llm_dllm": "automodel_amd.recipes.llm.train_dllm.TrainDiffusionLMRecipe",
}


def query_capabilities(arch: str | None = None) -> None:
    """Print per-model capability flags (reference cli/query_capabilities.py)."""
    from automodel_amd.models.common.capabilities import _CAPS, ModelCapabilities
    from automodel_amd.models.registry import _REGISTRY, _ensure_builtin

    _ensure_builtin()
    rows = [arch] if arch else sorted(set(list(_REGISTRY) + list(_CAPS)))
    for name in rows:
        cls = _REGISTRY.get(name)
        caps = _CAPS.get(cls.__name__ if cls else name, ModelCapabilities())
        flags = ", ".join(f"{k}={v}" for k, v in vars(caps).items())
        print(f"{name}: {flags}")


def generate_command(argv: list[str]) -> None:
    """Generate from a local checkpoint: one line of JSON per prompt. Prompts
    of any lengths run as batches through the cached decode path."""
    import argparse
    import json

    import torch

    from automodel_amd.models.registry import load_pretrained
    from automodel_amd.utils.generation import generate_batch

    ap = argparse.ArgumentParser(prog="automodel generate", description=generate_command.__doc__)
    ap.add_argument("--model", required=True, help="folder with config.json and safetensors")
    ap.add_argument("--prompt-ids", action="append", default=[], metavar="IDS",
                    help="comma-separated token ids; may be given several times")
    ap.add_argument("--prompt", action="append", default=[], metavar="TEXT",
                    help="text, with --tokenizer")
    ap.add_argument("--tokenizer", default=None, help="tokenizer folder")
    ap.add_argument("--max-new-tokens", type=int, default=32)
    ap.add_argument("--max-batch", type=int, default=16)
    ap.add_argument("--temperature", type=float, default=0.0)
    ap.add_argument("--eos", type=int, default=None, help="end token id")
    ap.add_argument("--dtype", default=None, choices=["bfloat16", "float32"])
    args = ap.parse_args(argv)

    tok = None
    if args.tokenizer:
        from automodel_amd.models.auto_tokenizer import build_tokenizer

        tok = build_tokenizer(args.tokenizer)
    if args.prompt and tok is None:
        ap.error("--prompt needs --tokenizer")
    prompts = [[int(t) for t in p.split(",")] for p in args.prompt_ids]
    prompts += [tok.encode(p) for p in args.prompt]
    if not prompts:
        ap.error("give --prompt-ids or --prompt")
    device = "cuda" if torch.cuda.is_available() else "cpu"
    dtype = args.dtype or ("bfloat16" if device == "cuda" else "float32")
    model = load_pretrained(args.model, dtype=dtype, device=device)
    outs = generate_batch(model, prompts, args.max_new_tokens, args.temperature, args.eos,
                          args.max_batch)
    for p, o in zip(prompts, outs):
        rec = {"prompt_ids": p, "output_ids": o}
        if tok is not None:
            rec["text"] = tok.decode(o)
        print(json.dumps(rec))


def main(argv: list[str] | None = None) -> None:
    argv = argv if argv is not None else sys.argv[1:]
    if not argv or argv[0] in ("-h", "--help"):
        print(__doc__)
        return
    if argv[0] == "capabilities":
        query_capabilities(argv[1] if len(argv) > 1 else None)
        return
    if argv[0] == "generate":
        generate_command(argv[1:])
        return
    cfg_path = argv[0]
    rest = argv[1:]
    nproc = 1
    if "--nproc-per-node" in rest:
        i = rest.index("--nproc-per-node")
        nproc = int(rest[i + 1])
        rest = rest[:i] + rest[i + 2:]
    overrides = parse_cli_overrides(rest)

    cfg = load_yaml_config(cfg_path)
    apply_overrides(cfg, overrides)
    recipe_name = cfg.get("recipe", "llm_finetune")
    target = RECIPE_ALIASES.get(recipe_name, recipe_name)

    from automodel_amd.launcher.interactive import InteractiveLauncher

    InteractiveLauncher(nproc_per_node=nproc).launch(cfg_path, target, rest)


if __name__ == "__main__":
    main()
