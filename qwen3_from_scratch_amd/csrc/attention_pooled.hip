// The paged attention kernels of attention.hip once more, for rows that see a window of tokens and,
// beside them, the means of the runs of tokens that have left it (see `RunSource` there): both sources
// go through the same tiles into one softmax. Only the matrix-core kernels are built here.
#define Q3_POOLED 1
#include "attention.hip"
