// Replays a request trace through a model: given token ids in, logits out, nothing sampled.
#pragma once
#include <cstddef>
#include <istream>
#include <string>

#include "model.h"

namespace cera {

// Steps come from `in`, one JSON object a line:
//   {"step": n, "entries": [{"id": name, "tokens": [...], "want": [places among these tokens]}], "end": [names]}
// The wanted logits of a step go to out_dir/<step>.f32 (little-endian f32, [wanted][vocab], in the order of
// the entries and of want); after every step a line "done <step>" is printed and flushed.  A step continues
// each request from what its earlier steps left; while several are alive the model's state is swapped between
// them by snapshots.  Throws BackendError.
void replay_trace(Model& model, std::istream& in, const std::string& out_dir);

// The command: --model DIR --out DIR [--dtype bfloat16|float32] [--max-tokens N] [--device D]; the exit code
int trace_main(int argc, char** argv, int first);

}  // namespace cera
