// Matrix-core attention whose scores fall with the distance, heads of up to 96 coordinates (see attention_mfma.inc).
#define ATTN_DISTANCE
#define DPAD 96
#include "attention_mfma.inc"
