// Matrix-core attention whose scores fall with the distance, heads of up to 64 coordinates (see attention_mfma.inc).
#define ATTN_DISTANCE
#define DPAD 64
#include "attention_mfma.inc"
