// The chunked recurrences (recurrence_chunks.h) whose decays are constants or formed from the projections as they are read
// (modes 0 to 2), and the entry point of all of them.
#include "recurrence_chunks.h"

int qe_recurrence_chunks_given(const Rec& a, hipStream_t stream);      // modes 3 to 5

// As qe_linear_recurrence (recurrence.hip), for rows cut into chunks on the host.  ws: float32, n_chunks * H *
// (D * Dv + D, in mode 5 + 2 D) numbers (not read if all_single: every portion is one chunk).  norm_w (heads of at most 128
// value columns): the normed and gated rows go to y instead of out.  Rows that no chunk names are left alone.
extern "C" int qe_linear_recurrence_chunked(const Rec* rec, hipStream_t stream) {
    const Rec& a = *rec;
    QE_REQUIRE(a.n_chunks >= 0 && a.n_portions >= 0, "linear_recurrence: bad sizes");
    QE_REC_CHECK(a, "linear_recurrence", false);
    QE_REQUIRE(a.D >= 4, "linear_recurrence: heads of %d key channels (4 to 256 in chunks)", a.D);
    if (a.n_chunks == 0) return 0;
    QE_REQUIRE(a.chunks && a.portions && (a.all_single || a.ws), "linear_recurrence: chunks without a workspace");
    QE_REQUIRE(a.row_stride < (1L << 23) && a.w_stride < (1L << 23) && (long)a.H * a.Dv < (1L << 23), "linear_recurrence: rows too long");
    QE_REQUIRE(a.norm_w ? a.Dv <= 128 : a.out != nullptr, "linear_recurrence: no place for the outputs, or heads too wide for the norm inside");
    if (a.mode >= 3) return qe_recurrence_chunks_given(a, stream);
#define QE_RP(TA_) (a.mode == 0 ? launch_phases<TA_, 0>(a, stream) : a.mode == 1 ? launch_phases<TA_, 1>(a, stream) : launch_phases<TA_, 2>(a, stream))
    return a.dt_a == QE_F32 ? QE_RP(float) : QE_RP(bf16_t);
#undef QE_RP
}
