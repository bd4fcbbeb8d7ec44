// The chunked recurrences (recurrence_chunks.h) whose decays were formed beforehand (modes 3 to 5).
#include "recurrence_chunks.h"

int qe_recurrence_chunks_given(const Rec& a, hipStream_t stream) {
#define QE_RP(TA_) (a.mode == 3 ? launch_phases<TA_, 3>(a, stream) : a.mode == 4 ? launch_phases<TA_, 4>(a, stream) : launch_phases<TA_, 5>(a, stream))
    return a.dt_a == QE_F32 ? QE_RP(float) : QE_RP(bf16_t);
#undef QE_RP
}
