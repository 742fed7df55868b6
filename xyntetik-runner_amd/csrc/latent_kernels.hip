// Attention whose keys and values are made from one small latent a token ("latent attention").
//
// What is cached a token is one row [c (C channels) | k_rot (R channels)]: the normed latent and
// the rotated key part that all heads share.  Queries are brought into the latent's space (per
// head q_abs = W_uk^T q_unrotated, a product of its own), so a head's score over the cached row is
//     q_abs . c + q_rot . k_rot     = q_unrotated . (W_uk c) + q_rot . k_rot,
// attention runs as one key/value head of size C + R shared by all query heads, its value is the
// latent itself, and W_uv is applied to the attention's output.  k_latent_prepare does everything
// between the two down projections and the attention: the latent's RMSNorm, the rotation of the
// shared key part and of every head's rotated query channels (the first `dims` of the R channels, in pairs
// (2i, 2i+1) or, with `halves`, (i, i + dims/2); angle = position x inv_freq[i] formed in 32 bits), the write of the cached
// row into the key pages [page][0][slot][C + R] and, transposed, into the value pages
// [page][0][Dvc][slot] (Dvc = C, or C + R where the attention kernel wants values as long as
// keys), and the copy of the unrotated query channels in the compute type for the product that
// follows.  Without kv_in (a layer that reads another layer's rows) only the queries are made.  A workgroup a token.
#include "common.h"

template <typename TO, int NW>
__global__ __launch_bounds__(64 * NW) void k_latent_prepare(
    TO* __restrict__ qn_out, TO* __restrict__ q_out, TO* __restrict__ k_cache, TO* __restrict__ v_cache,
    const float* __restrict__ q_in, const float* __restrict__ kv_in, const float* __restrict__ c_w,
    const int* __restrict__ positions, const int* __restrict__ req_of_token, const int* __restrict__ block_table,
    const float* __restrict__ inv_freq, int table_stride, int H, int D, int R, int C, int Dvc, int dims, int halves, int ld_q, int ld_kv,
    int page_shift, int page_size, float eps) {
    constexpr int NT = 64 * NW;
    __shared__ float part[NW];
    const int t = blockIdx.x, tid = threadIdx.x;
    const int pos = positions[t];
    const float* kv = kv_in + (kv_in ? (size_t)t * ld_kv : 0);
    const int DK = C + R;
    TO *krow = nullptr, *vpage = nullptr;
    if (kv_in) {
        // the latent's norm
        float ss = 0.f;
        for (int i = tid; i < C; i += NT) ss += kv[i] * kv[i];
        ss = wave_sum(ss);
        if ((tid & 63) == 0) part[tid >> 6] = ss;
        __syncthreads();
        float tot = 0.f;
#pragma unroll
        for (int i = 0; i < NW; ++i) tot += part[i];
        const float rinv = 1.0f / sqrtf(tot / (float)C + eps);
        const PageRef pr = page_of(block_table, table_stride, req_of_token[t], pos, page_shift, page_size - 1);
        krow = k_cache + ((size_t)pr.page * page_size + pr.off) * DK;
        vpage = v_cache + (size_t)pr.page * Dvc * page_size + pr.off;
        for (int i = tid; i < C; i += NT) {
            const float c = kv[i] * rinv * c_w[i];
            st<TO>(krow, i, c);
            st<TO>(vpage, (size_t)i * page_size, c);
        }
    }
    // the shared key part and every head's rotated query channels: unit u = 0 is the key, u = 1 + h head h
    const int half = dims >> 1, pairs_r = (R + 1) >> 1;       // a "pair" past `dims` is two channels that pass unchanged
    for (int w = tid + (kv_in ? 0 : pairs_r); w < (H + 1) * pairs_r; w += NT) {
        const int u = w / pairs_r, i = w - u * pairs_r;
        const float* src = u == 0 ? kv + C : q_in + (size_t)t * ld_q + (size_t)(u - 1) * (D + R) + D;
        const int c0 = halves && i < half ? i : 2 * i, c1 = halves && i < half ? i + half : 2 * i + 1;
        float a = src[c0], b = c1 < R ? src[c1] : 0.f;
        if (i < half) {
            const float ang = (float)pos * inv_freq[i];
            const float cs = cosf(ang), sn = sinf(ang);
            const float ra = a * cs - b * sn, rb = b * cs + a * sn;
            a = ra;
            b = rb;
        }
        if (u == 0) {
            st<TO>(krow, C + c0, a);
            if (c1 < R) st<TO>(krow, C + c1, b);
            if (Dvc > C) {
                st<TO>(vpage, (size_t)(C + c0) * page_size, a);
                if (c1 < R) st<TO>(vpage, (size_t)(C + c1) * page_size, b);
            }
        } else {
            TO* dst = q_out + ((size_t)t * H + (u - 1)) * DK + C;
            st<TO>(dst, c0, a);
            if (c1 < R) st<TO>(dst, c1, b);
        }
    }
    // the unrotated query channels, head by head, for the product into the latent's space
    for (int w = tid; w < H * D; w += NT) {
        const int h = w / D, d = w - h * D;
        st<TO>(qn_out, (size_t)t * H * D + w, q_in[(size_t)t * ld_q + (size_t)h * (D + R) + d]);
    }
}

extern "C" int xr_latent_prepare(void* qn_out, void* q_out, void* k_cache, void* v_cache, const float* q_in, const float* kv_in,
                                 const float* c_w, const int* positions, const int* req_of_token, const int* block_table,
                                 int table_stride, const float* inv_freq, int T, int H, int D, int R, int C, int Dvc, int dims,
                                 int halves, int ld_q, int ld_kv, int page_size, float eps, int dtype, hipStream_t stream) {
    XR_REQUIRE(T >= 0 && H > 0 && D > 0 && R >= 0 && C > 0, "latent_prepare: bad sizes T=%d H=%d D=%d R=%d C=%d", T, H, D, R, C);
    XR_REQUIRE(Dvc == C || Dvc == C + R, "latent_prepare: values of %d channels (the latent's %d, or %d with the rotated part)", Dvc, C, C + R);
    XR_REQUIRE(dims >= 0 && dims % 2 == 0 && dims <= R && (dims == 0 || inv_freq), "latent_prepare: %d rotated channels of %d", dims, R);
    XR_REQUIRE(ld_q >= H * (D + R) && (!kv_in || ld_kv >= C + R), "latent_prepare: row strides %d, %d are too short", ld_q, ld_kv);
    const int shift = ilog2_exact(page_size);
    XR_REQUIRE(shift >= 0, "latent_prepare: page size %d is no power of two", page_size);
    if (T == 0) return XR_OK;
#define LP(TO, NW)                                                                                                            \
    k_latent_prepare<TO, NW><<<T, 64 * NW, 0, stream>>>((TO*)qn_out, (TO*)q_out, (TO*)k_cache, (TO*)v_cache, q_in, kv_in, c_w,  \
                                                        positions, req_of_token, block_table, inv_freq, table_stride, H, D, R, \
                                                        C, Dvc, dims, halves, ld_q, ld_kv, shift, page_size, eps)
    // (a decode step's few rows: their time is the latency of one workgroup's passes)
    const bool few = T <= 128 && H * (D + R) >= 1024;
    if (dtype == XR_F32) { if (few) LP(float, 16); else LP(float, 4); }
    else if (dtype == XR_BF16) { if (few) LP(bf16_t, 16); else LP(bf16_t, 4); }
    else { xr_set_error("latent_prepare: bad dtype %d", dtype); return XR_BAD_ARG; }
#undef LP
    XR_CHECK_LAUNCH("latent_prepare");
    return XR_OK;
}
