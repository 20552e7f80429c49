// The trace runner as a program of its own: the directory models only, so it needs neither the
// block-quantized kernels nor the GGUF layer.  `cera-hip trace` is the same command.
#include "trace.h"

int main(int argc, char** argv) { return cera::trace_main(argc, argv, 1); }
