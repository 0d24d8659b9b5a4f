"""Trace replay: feed given token ids through a model step by step and write the logits that are asked for (bin/trace_run). Steps arrive on standard input, one JSON
object per line - {"step": n, "entries": [{"id", "tokens", "want"}], "end": [ids]} -; every step is one engine batch, and "done n" follows it on standard output."""
import argparse
import json
import os
import sys


def build_if_missing():
    """compile what dense-weight models need when no library is built yet"""
    from . import lib
    if not os.path.exists(lib.lib_path()):
        from . import build
        build.build_dense()


class Replay:
    def __init__(self, model, out):
        self.model, self.out, self.seqs = model, out, {}

    def step(self, msg):
        import torch
        entries = []
        for e in msg["entries"]:
            if not e["tokens"]:
                continue
            if e["id"] not in self.seqs:
                self.seqs[e["id"]] = self.model.seq_new()
            entries.append((self.seqs[e["id"]], e["tokens"], e["want"]))
        rows = sum(len(w) for _, _, w in entries)
        logits = torch.empty(rows, self.model.n_vocab, dtype=torch.float32, device=self.model.dev) if rows else None
        if entries:
            self.model.batch(entries, logits=logits)
        if rows:
            part = os.path.join(self.out, "%d.f32.part" % msg["step"])
            logits.cpu().numpy().astype("<f4").tofile(part)
            os.replace(part, part[:-len(".part")])
        for i in msg.get("end", ()):
            if i in self.seqs:
                self.model.seq_free(self.seqs.pop(i))


def main(argv=None):
    ap = argparse.ArgumentParser(prog="trace_run", description="replay a trace of token ids through a model and write the wanted logits")
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", default="bfloat16", choices=("bfloat16", "float32"))
    ap.add_argument("--out", required=True, help="folder for <step>.f32")
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens that live requests hold, each rounded up to 64")
    ap.add_argument("--max-requests", type=int, default=4, help="most live requests")
    ap.add_argument("--pass-tokens", type=int, default=4096, help="tokens per pass over the layers; longer steps run in pieces")
    a = ap.parse_args(argv)
    stdout = os.fdopen(os.dup(1), "w")
    os.dup2(2, 1)                                         # (whatever a compiler prints does not belong among the answers)
    build_if_missing()
    from . import registry
    model = registry.load(a.model, dtype=a.dtype)
    model.finalize_pool(min(a.max_tokens, a.pass_tokens), a.max_requests, a.max_tokens)
    replay = Replay(model, a.out)
    for line in sys.stdin:
        if not line.strip():
            continue
        msg = json.loads(line)
        replay.step(msg)
        stdout.write("done %d\n" % msg["step"])
        stdout.flush()
    model.close()
    return 0
