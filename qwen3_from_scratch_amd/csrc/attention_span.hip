// The paged attention kernels of attention.hip once more, for rows that see a span of the tokens before:
// a chunk of the sequence, or a window and the sequence's first tokens (see `Span` there), with keys and
// values that may differ in size. Only the matrix-core kernels are built here.
#define Q3_SPAN 1
#include "attention.hip"
