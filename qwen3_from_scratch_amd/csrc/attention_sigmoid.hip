// The paged attention kernels of attention.hip once more, for keys that count by the sigmoid of their
// biased scores, without a softmax (see Q3_SIGMOID there). Only the matrix-core kernels are built here.
#define Q3_SIGMOID 1
#include "attention.hip"
