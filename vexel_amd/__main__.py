"""Command line of the engine.

  python -m vexel_amd generate --model PATH --tokens 5,17,3 [--tokens ..] [--max-new 16] [--dtype bfloat16|float32]
                               [--temperature T --top-k K --top-p P --seed S] [--prefill-chunk N] [--eos ID]
  python -m vexel_amd architectures

generate: PATH is a folder with config.json and model.safetensors or a GGUF file. Each --tokens is one request (token
ids; there is no tokenizer here); all of them run together through the scheduler. One line of generated ids is printed
per request, in their order. architectures: what a folder's config.json may name."""
import argparse
import sys


def generate(a):
    from .backend import HipBackend
    from .runtime import ModelRuntime, Scheduler
    prompts = [[int(t) for t in p.replace(",", " ").split()] for p in a.tokens]
    blocks = [(len(p) + a.max_new + a.block_size - 1) // a.block_size + 1 for p in prompts]
    be = HipBackend(a.device)
    mr = ModelRuntime.load(be, a.model, dtype=a.dtype, block_size=a.block_size, pool_blocks=sum(blocks), max_seqs=len(prompts),
                           max_blocks_per_seq=max(blocks), max_batch=max(len(prompts), a.prefill_chunk, 1))
    s = Scheduler(mr, len(prompts), a.max_new, a.eos, a.prefill_chunk)
    for i, p in enumerate(prompts):
        s.add_sequence(i, p)
        if a.temperature > 0:
            s.set_sampling(i, a.temperature, a.top_k, a.top_p, a.seed + i)
    FINISHED = 3
    while any(s.state(i) != FINISHED for i in range(len(prompts))):
        s.step()
    for i in range(len(prompts)):
        print(" ".join(str(t) for t in s.generated(i)))
    s.close()
    mr.close()
    be.close()


def main(argv=None):
    ap = argparse.ArgumentParser(prog="python -m vexel_amd", description=__doc__,
                                 formatter_class=argparse.RawDescriptionHelpFormatter)
    sub = ap.add_subparsers(dest="command", required=True)
    g = sub.add_parser("generate", help="generate from token ids")
    g.add_argument("--model", required=True)
    g.add_argument("--tokens", action="append", required=True, help="a request's token ids, comma-separated; repeatable")
    g.add_argument("--max-new", type=int, default=16)
    g.add_argument("--dtype", choices=["bfloat16", "float32"], default=None, help="activations of a folder's model")
    g.add_argument("--temperature", type=float, default=0.0)
    g.add_argument("--top-k", type=int, default=0)
    g.add_argument("--top-p", type=float, default=0.0)
    g.add_argument("--seed", type=int, default=0)
    g.add_argument("--eos", type=int, default=-1)
    g.add_argument("--prefill-chunk", type=int, default=0, help="tokens of a prompt per step, 0 = all")
    g.add_argument("--block-size", type=int, default=16)
    g.add_argument("--device", type=int, default=0)
    sub.add_parser("architectures", help="list what config.json may name")
    a = ap.parse_args(argv)
    if a.command == "architectures":
        from .runtime import architectures
        print("\n".join(architectures()))
    else:
        generate(a)
    return 0


if __name__ == "__main__":
    sys.exit(main())
