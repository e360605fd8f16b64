// The matrix-core attention kernels of attention_mfma.hip once more, with a cap on the scores: a scaled score s becomes
// softcap * tanh(s / softcap).  Every entry point takes, as its last argument, softcap (positive).  A library of its
// own, so that the kernels without a cap carry nothing for it.
#define LCU_SCORE_CAP 1
#include "attention_mfma.hip"
