// What the attention launches make of a PtaScoreBias (pta_kernels.h): one of the three ways the kernels form the
// bias, or a refusal by name; and of a PtaHeadRows.
#pragma once

#include "common.h"
#include "pta_kernels.h"

// mode: 0 slope x key position with the position and the product rounded to bfloat16, 1 the same exact, 2 slope x
// (key position - query position) exact.  Returns 0, or nonzero with the reason in pta_last_error.
static inline int pta_score_bias_mode(const char* what, const PtaScoreBias* b, int* mode) {
    *mode = 1;
    if (!b || !b->slopes) return 0;
    PTA_REQUIRE(b->of == PTA_BIAS_KEY || b->of == PTA_BIAS_DISTANCE,
                "%s: a score bias of kind %d is not built; built are slope x key position and slope x (key position - "
                "query position), one slope per head", what, b->of);
    PTA_REQUIRE(!b->bf16 || b->of == PTA_BIAS_KEY,
                "%s: rounding to bfloat16 as the reference rounds is built for slope x key position only", what);
    *mode = b->of == PTA_BIAS_DISTANCE ? 2 : b->bf16 ? 0 : 1;
    return 0;
}

// where the heads go, as a launch takes it (PtaHeadRows, pta_kernels.h)
static inline PtaHeadRows pta_head_rows_of(const PtaHeadRows* given, int nh, int d) {
    return given ? *given : PtaHeadRows{(long)nh * d, d, d, 1.0f};
}
static inline int pta_check_head_rows(const char* what, const PtaHeadRows& r, int nh, int d, const void* out, int vec) {
    PTA_REQUIRE(r.keep > 0 && r.keep <= d && r.head >= r.keep && r.ld >= (long)(nh - 1) * r.head + r.keep,
                "%s: %d elements of every head, heads %d apart in rows %ld apart, overlap or are more than a head has", what, r.keep,
                r.head, r.ld);
    PTA_REQUIRE(r.keep % vec == 0 && r.head % vec == 0 && r.ld % vec == 0 && ((uintptr_t)out % (2 * vec)) == 0,
                "%s: heads are written %d elements at a time, and their places must be multiples of that", what, vec);
    return 0;
}
