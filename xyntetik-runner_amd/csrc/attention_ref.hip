// Attention over the paged cache with 32-bit arithmetic only: the attention of the
// true 32-bit path, for prompt portions and decoded tokens alike, any head size up
// to 256.  One wave per (token, query head).
//
// For the token at position p of its request and query head h (key/value head
// h / (H/Hk), contiguous groups): s_t = (q . K_t) * scale for t in [lo, p], causal by
// the loop bound, lo = max(0, p - window + 1) for a windowed layer
// (src/model.c:3553-3573, :6326); softmax with the maximum taken out
// (src/model.c:3409-3415); out = sum_t p_t V_t (:3576-3587).  The
// softmax runs over blocks of 64 keys with a running maximum and sum, which gives the
// same value up to rounding.  With `slopes` (one number a query head) a bias that grows with the distance is
// taken off every score: s_t = (q . K_t) * scale - slope_h * (p - t).
// Other masks: `chunk` > 0: lo = p - p mod chunk (a position reads its own chunk of positions, counted from 0);
// `keep` > 0: the keys [0, keep) are read as well wherever lo lies.  `sinks` (one number a query head): the
// softmax's denominator also holds exp(sink_h) (of the sink as it is: no scale, no cap), an entry that has no key and no value.  Values may have another
// size than keys (Dv; cache layout K [page][kv_head][slot][D], V [page][kv_head][Dv][slot]).
// With `cap` > 0 a scaled score s counts as cap * tanh(s / cap), before a slope's bias.  A head's output is multiplied by
// `out_scale` and, with `gate` (a number a token and head), by sigmoid(gate); output rows are ld_out apart.
#include "common.h"

#define AR_MAX_D 256

template <typename T>
__global__ __launch_bounds__(64) void k_attention_ref(
    T* __restrict__ out, const T* __restrict__ q, const T* __restrict__ kc, const T* __restrict__ vc,
    const int* __restrict__ positions, const int* __restrict__ req_of_token,
    const int* __restrict__ block_table, int table_stride, int H, int Hk, int D, int Dv, int page_shift,
    int page_mask, int page_size, float scale, int window, int chunk, int keep, const float* __restrict__ slopes,
    const float* __restrict__ sinks, float cap, const float* __restrict__ gate, int ld_gate, float out_scale, int ld_out) {
    __shared__ float qs[AR_MAX_D];
    const int t = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
    const int pos = positions[t];
    const int req = req_of_token[t];
    const int kvh = h / (H / Hk);
    const int lo = chunk > 0 ? pos - pos % chunk : (window > 0 && pos - window + 1 > 0) ? pos - window + 1 : 0;
    const int kept = keep < lo ? keep : lo;         // kept keys [0, kept) lie below the row's own range
    const T* qrow = q + ((size_t)t * H + h) * D;
    for (int d = lane; d < D; d += 64) qs[d] = ld<T>(qrow, d);
    __syncthreads();
    const int* bt = block_table + (size_t)req * table_stride;
    const float slope = slopes ? slopes[h] : 0.f;

    float m = -INFINITY, l = 0.f;
    float acc[AR_MAX_D / 64];
#pragma unroll
    for (int dd = 0; dd < AR_MAX_D / 64; ++dd) acc[dd] = 0.f;

    for (int seg = kept > 0 ? 0 : 1; seg < 2; ++seg)
    for (int k0 = seg ? lo : 0, last = seg ? pos : kept - 1; k0 <= last; k0 += 64) {
        const int key = k0 + lane;
        const bool valid = key <= last;
        float s = -INFINITY;
        if (valid) {
            const int page = bt[key >> page_shift];
            const int off = key & page_mask;
            const T* kr = kc + (((size_t)page * Hk + kvh) * page_size + off) * D;
            float dot = 0.f;
            for (int d = 0; d < D; ++d) dot = fmaf(qs[d], ld<T>(kr, d), dot);
            s = dot * scale;
            if (cap > 0.f) s = cap * tanhf(s / cap);
            s -= slope * (float)(pos - key);
        }
        const float mn = fmaxf(m, wave_max(s));
        const float p = valid ? expf(s - mn) : 0.f;
        const float corr = m == -INFINITY ? 0.f : expf(m - mn);
        l = l * corr + wave_sum(p);
#pragma unroll
        for (int dd = 0; dd < AR_MAX_D / 64; ++dd) acc[dd] *= corr;
        const int nk = (last - k0 + 1) < 64 ? (last - k0 + 1) : 64;
        for (int j = 0; j < nk; ++j) {
            const float pj = __shfl(p, j, 64);
            const int kj = k0 + j;
            const int page = bt[kj >> page_shift];
            const int off = kj & page_mask;
            const T* vb = vc + ((size_t)page * Hk + kvh) * Dv * page_size + off;
#pragma unroll
            for (int dd = 0; dd < AR_MAX_D / 64; ++dd) {
                const int d = lane + 64 * dd;
                if (d < Dv) acc[dd] = fmaf(pj, ld<T>(vb, (size_t)d * page_size), acc[dd]);
            }
        }
        m = mn;
    }
    if (sinks) {            // one more entry of the denominator, with nothing to add to the output
        const float sk = sinks[h];
        const float mn = fmaxf(m, sk);
        const float corr = expf(m - mn);
        l = l * corr + expf(sk - mn);
#pragma unroll
        for (int dd = 0; dd < AR_MAX_D / 64; ++dd) acc[dd] *= corr;
    }
    T* orow = out + (size_t)t * ld_out + (size_t)h * Dv;
    const float f = gate ? out_scale / (1.0f + expf(-gate[(size_t)t * ld_gate + h])) : out_scale;
#pragma unroll
    for (int dd = 0; dd < AR_MAX_D / 64; ++dd) {
        const int d = lane + 64 * dd;
        if (d < Dv) st<T>(orow, d, acc[dd] / l * f);
    }
}

extern "C" int xr_attention_ref(void* out, const void* q, const void* k_cache, const void* v_cache,
                                const int* positions, const int* req_of_token, const int* block_table,
                                int table_stride, int T, int H, int Hk, int D, int Dv, int page_size, float scale,
                                int window, int chunk, int keep, int dtype, const float* slopes, const float* sinks,
                                float cap, const float* gate, int ld_gate, float out_scale, int ld_out, hipStream_t stream) {
    XR_REQUIRE(ld_out >= H * Dv && (!gate || ld_gate >= H), "attention: output rows %d apart, gate rows %d apart for %d heads of %d", ld_out, ld_gate, H, Dv);
    XR_REQUIRE(cap >= 0.f, "attention: soft cap %g of the scores is negative", (double)cap);
    XR_REQUIRE(T >= 0 && H > 0 && Hk > 0 && D > 0, "attention: bad sizes T=%d H=%d Hk=%d D=%d", T, H, Hk, D);
    XR_REQUIRE(H % Hk == 0, "attention: %d query heads are not a multiple of %d key/value heads", H, Hk);
    XR_REQUIRE(D <= AR_MAX_D && Dv > 0 && Dv <= AR_MAX_D, "attention: head size %d or value size %d exceeds %d", D, Dv, AR_MAX_D);
    XR_REQUIRE(chunk >= 0 && keep >= 0, "attention: chunk %d or kept keys %d are negative", chunk, keep);
    int shift = ilog2_exact(page_size);
    XR_REQUIRE(shift >= 0, "attention: page size %d is not a power of two", page_size);
    XR_REQUIRE(window >= 0, "attention: window %d is negative", window);
    if (T == 0) return XR_OK;
    dim3 grid(T, H);
    if (dtype == XR_F32)
        k_attention_ref<float><<<grid, 64, 0, stream>>>((float*)out, (const float*)q, (const float*)k_cache,
                                                        (const float*)v_cache, positions, req_of_token, block_table,
                                                        table_stride, H, Hk, D, Dv, shift, page_size - 1, page_size, scale, window, chunk, keep, slopes, sinks, cap, gate, ld_gate, out_scale, ld_out);
    else if (dtype == XR_BF16)
        k_attention_ref<bf16_t><<<grid, 64, 0, stream>>>((bf16_t*)out, (const bf16_t*)q, (const bf16_t*)k_cache,
                                                         (const bf16_t*)v_cache, positions, req_of_token, block_table,
                                                         table_stride, H, Hk, D, Dv, shift, page_size - 1, page_size, scale, window, chunk, keep, slopes, sinks, cap, gate, ld_gate, out_scale, ld_out);
    else { xr_set_error("attention: bad dtype %d", dtype); return XR_BAD_ARG; }
    XR_CHECK_LAUNCH("attention_ref");
    return XR_OK;
}
