// Decode step (one token) of a parallel-residual layer of a layer-list decoder in three launches (five with latent
// attention): the normed projections (fh_matvec_norm), this file's middle launch - the mixer's own step beside the routed
// experts' gate and up products - and the output launch, which adds every down-stream product of the layer into the
// residual stream:  x += W_o . mix + sum_j w_j D_(e_j) . a_j + D_s . a_s.
#pragma once
#include "fh_gqa.h"
#include "fh_latent.h"
#include "fh_moe.h"

enum { FH_MIX_RECURRENT = 0, FH_MIX_LATENT = 1 };
struct FhStep {
    int kind = 0;              // FH_MIX_*
    FhRecurrent rec;
    FhRecState rec_state;
    FhLatent lat;
    const float *proj = nullptr; // this token's projection row
    const float *hn = nullptr;   // the layer's normed input [kp]
    int kp = 0;                  // input length of the experts, padded
    const int *pos_dev = nullptr;
    float *qa = nullptr;         // absorbed queries (latent)
    float *o = nullptr;          // output of the mixer before its gate, norm and output projection [heads * vdim]
    FhMoe moe;
    float *act = nullptr;        // [top, ffp] expert activations
    int *ids = nullptr;          // [top]
    float *wts = nullptr;        // [top]
    const float *s_gu = nullptr; // gate and up products of the always-on expert [2 sffp]
    const uint16_t *wo = nullptr; // [width, kpo]
    int kpo = 0, width = 0;
    float *x = nullptr;          // residual stream
};
fh_status fh_step_middle(fh_device *dev, int dtype, const FhStep &st, fh_kvcache *cache);
fh_status fh_step_out(fh_device *dev, const FhStep &st);

// A layer whose sublayers are normed at their end keeps them apart, each a chain of its own:
//   projections (fh_matvec_mix: the sublayer before is normed and added on the way in) - fh_step_mixers: attention over parts
//   of the cache beside the recurrence's step - fh_step_mix_out: merge of the parts, norm and gate of the recurrence -
//   output projection (fh_matvec_mix) - feed-forward (twice fh_matvec_mix)
// `act` is the input of the output projection: the attention's heads * vdim values padded to kpl with zeros, then the
// recurrence's.
struct FhMixStep {
    int attn = 0, rec = 0;       // which mixers there are
    FhGqa gqa;
    FhRecurrent r;
    FhRecState state;
    const float *proj = nullptr; // this token's projection row
    const int *pos_dev = nullptr;
    float *part = nullptr, *o = nullptr, *act = nullptr;
    int kpl = 0;
};
fh_status fh_step_mixers(fh_device *dev, int dtype, const FhMixStep &st, fh_kvcache *cache);
fh_status fh_step_mix_out(fh_device *dev, const FhMixStep &st, const fh_kvcache *cache);
