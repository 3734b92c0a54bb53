#include "talking.h"
bool pa_talking_prefill_launch(const TalkArgs &, int, hipStream_t, int &) { return false; }
