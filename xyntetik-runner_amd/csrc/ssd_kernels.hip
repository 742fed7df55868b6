// A selective state space with one decay a token and head over long portions, in chunks on the matrix cores.
//
//   S_t = exp(-a dt_t) S_(t-1) + dt_t B_t x_t^T;   y_t = S_t^T C_t + D x_t        (S is [N, Dv])
//
// is a chain only through the state before a chunk.  With c_i the sum of -a dt_t over a chunk's rows up to i (inclusive):
//
//   y_i = exp(c_i) S_before^T C_i + sum_(j <= i) exp(c_i - c_j) dt_j (C_i . B_j) x_j + D x_i
//   S_after = exp(c_last) S_before + sum_j exp(c_last - c_j) dt_j B_j x_j^T
//
// so three launches do a portion of any length:
//   k_ssd_state   every chunk's own sum over j (as if the state before it were zero) and exp(c_last);
//   k_ssd_carry   one element of a head's state a thread, chunk after chunk: the state before every chunk, in place,
//                 and the request's new state;
//   k_ssd_out     the read-outs.
// x, B and C come as the convolution leaves them, rounded to bfloat16.  Everything that multiplies them is 32-bit and goes
// to the matrix cores as two bfloat16 numbers, high and low part, in two products that add up in 32 bits: the scaled rows
// dt_j exp(c_last - c_j) x_j, the state before a chunk, and the weights exp(c_i - c_j) dt_j (C_i . B_j).  The sums c are
// formed and subtracted in 64 bits (a chunk's sum may be thousands where neighbours differ by hundredths).
//
// The host lists the chunks (request, first row, rows) of at most 128 rows; the states of the chunks lie as a request's
// state does (recurrent_kernels.hip): S[n][v] of a head at ((n / R) Dv + v) R + n % R, rows from N to the next multiple of
// R zero.  As in the attention kernels the products are arranged so that a lane keeps one row i: G^T[j, i] = B_j . C_i has
// row i in a lane's column, and with the rows of a tile of 32 j permuted (key_off) the 8 weights a lane holds for 16 j are
// the 8 the next product takes from it as operand.
#include "common.h"

typedef __bf16 sd_bf16x8 __attribute__((ext_vector_type(8)));
typedef float sd_f32x16 __attribute__((ext_vector_type(16)));

#define SSD_L 128           // rows of a chunk
#define SSD_V 64            // channels of x a workgroup takes
#define SSD_LD (SSD_L + 8)  // LDS elements between rows that hold a chunk's tokens

struct SsdArgs {
    float* out;             // [T, H * Dv]
    const bf16_t* x;        // [T, ld]: H heads of Dv
    const bf16_t* b;        // [T, ld]: G groups of N
    const bf16_t* c;        // [T, ld]: G groups of N
    const float* z;         // [T, ld_z]: the step sizes' projections, H of them
    const float* constants; // [3][H]: a, the step sizes' bias, D
    float* state;           // [slots, H, J, Dv, R]
    float* scratch;         // [items, H, J, Dv, R]
    float* prod;            // [items, H]
    const int* items;       // [n_items, 4]: request, first row, rows, -
    const int* requests;    // [B, 2]: first item, items
    const int* slots;
    int H, G, N, Dv, R, ld, ld_z;
};

__device__ inline sd_bf16x8 sd_frag(uint4 v) {
    union { uint4 u; sd_bf16x8 b; } c;
    c.u = v;
    return c.b;
}
// two floats as bfloat16 pairs: what rounding keeps, and what it leaves
__device__ inline void split2(float a, float b, uint32_t& hi, uint32_t& lo) {
    hi = pack_bf16x2(a, b);
    lo = pack_bf16x2(a - __uint_as_float(hi << 16), b - __uint_as_float(hi & 0xffff0000u));
}

// dt[j] and the inclusive sums cum[j] of -a dt over the chunk's rows (rows past the end: dt 0, the sum stays), by the
// first wave: two rows a lane.
__device__ inline void ssd_steps(const SsdArgs& a, int h, int row0, int rows, float* dt, double* cum) {
    if (threadIdx.x < 64) {
        const int lane = threadIdx.x;
        const float rate = a.constants[h], bias = a.constants[a.H + h];
        float d[2];
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            const int j = 2 * lane + u;
            const float z = j < rows ? a.z[(size_t)(row0 + j) * a.ld_z + h] + bias : 0.f;
            d[u] = j < rows ? (z > 20.0f ? z : log1pf(expf(z))) : 0.f;
            dt[j] = d[u];
        }
        const double l0 = -(double)rate * d[0], l1 = -(double)rate * d[1];
        double s = l0 + l1;
        for (int o = 1; o < 64; o <<= 1) {
            const double t = __shfl_up(s, o, 64);
            if (lane >= o) s += t;
        }
        cum[2 * lane] = s - l1;
        cum[2 * lane + 1] = s;
    }
    __syncthreads();
}

// A tile of rows [token][channel] of bfloat16 into LDS transposed, [channel][token]: a thread takes two tokens and 8
// channels, so that it writes pairs.  f(j, value) is applied on the way, both parts of it kept if `lo` is given.
template <class F>
__device__ inline void load_transposed(bf16_t* hi, bf16_t* lo, const bf16_t* src, int ld, int row0, int rows, int c_end, int groups, F f) {
    for (int q = threadIdx.x; q < groups * (SSD_L / 2); q += 256) {
        const int jp = q % (SSD_L / 2), c8 = q / (SSD_L / 2);
        const int j = 2 * jp, ch = c8 * 8;
        uint4 r0 = make_uint4(0, 0, 0, 0), r1 = r0;
        if (ch < c_end) {           // (a multiple of 8: all 8 channels exist)
            if (j < rows) r0 = *reinterpret_cast<const uint4*>(src + (size_t)(row0 + j) * ld + ch);
            if (j + 1 < rows) r1 = *reinterpret_cast<const uint4*>(src + (size_t)(row0 + j + 1) * ld + ch);
        }
        const uint32_t w0[4] = {r0.x, r0.y, r0.z, r0.w}, w1[4] = {r1.x, r1.y, r1.z, r1.w};
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const uint32_t a = (e & 1) ? w0[e >> 1] >> 16 : w0[e >> 1] & 0xffffu, b = (e & 1) ? w1[e >> 1] >> 16 : w1[e >> 1] & 0xffffu;
            uint32_t* dst = reinterpret_cast<uint32_t*>(hi + (size_t)(ch + e) * SSD_LD + j);
            if (lo) {
                uint32_t h2, l2;
                split2(f(j, __uint_as_float(a << 16)), f(j + 1, __uint_as_float(b << 16)), h2, l2);
                *dst = h2;
                *reinterpret_cast<uint32_t*>(lo + (size_t)(ch + e) * SSD_LD + j) = l2;
            } else {
                *dst = a | (b << 16);
            }
        }
    }
}

// NB: blocks of 32 state rows that the LDS holds
template <int NB>
__global__ __launch_bounds__(256) void k_ssd_state(SsdArgs a) {
    extern __shared__ __attribute__((aligned(16))) bf16_t lds[];
    bf16_t* xh = lds;                                   // [SSD_V][SSD_LD] the scaled rows, high parts
    bf16_t* xl = xh + SSD_V * SSD_LD;                   // low parts
    bf16_t* bt = xl + SSD_V * SSD_LD;                   // [32 NB][SSD_LD]
    __shared__ float dt[SSD_L];
    __shared__ double cum[SSD_L];
    const int item = blockIdx.z, h = blockIdx.y, v0 = blockIdx.x * SSD_V;
    const int row0 = a.items[item * 4 + 1], rows = a.items[item * 4 + 2];
    ssd_steps(a, h, row0, rows, dt, cum);
    const double last = cum[SSD_L - 1];
    const int g = h / (a.H / a.G);
    load_transposed(xh, xl, a.x + h * a.Dv + v0, a.ld, row0, rows, a.Dv - v0, SSD_V / 8,
                    [&](int j, float v) { return v * (dt[j] * expf((float)(last - cum[j]))); });
    load_transposed(bt, (bf16_t*)nullptr, a.b + g * a.N, a.ld, row0, rows, a.N, NB * 4, [](int, float v) { return v; });
    __syncthreads();
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, lr = lane & 31, lg = lane >> 5;
    const int J = (a.N + a.R - 1) / a.R;
    float* cp = a.scratch + ((size_t)item * a.H + h) * J * a.Dv * a.R;
    for (int nb = wave; nb < NB; nb += 4) {
        sd_f32x16 acc[2];
#pragma unroll
        for (int d = 0; d < 2; ++d)
#pragma unroll
            for (int e = 0; e < 16; ++e) acc[d][e] = 0.f;
#pragma unroll
        for (int ks = 0; ks < SSD_L / 16; ++ks) {
            const int j = ks * 16 + lg * 8;
            const sd_bf16x8 bf = sd_frag(*reinterpret_cast<const uint4*>(bt + (nb * 32 + lr) * SSD_LD + j));
#pragma unroll
            for (int d = 0; d < 2; ++d) {
                const sd_bf16x8 ah = sd_frag(*reinterpret_cast<const uint4*>(xh + (d * 32 + lr) * SSD_LD + j));
                const sd_bf16x8 al = sd_frag(*reinterpret_cast<const uint4*>(xl + (d * 32 + lr) * SSD_LD + j));
                acc[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(ah, bf, acc[d], 0, 0, 0);
                acc[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(al, bf, acc[d], 0, 0, 0);
            }
        }
        const int n = nb * 32 + lr;
        if (n >= J * a.R) continue;
        float* col = cp + ((size_t)(n / a.R) * a.Dv) * a.R + n % a.R;
#pragma unroll
        for (int d = 0; d < 2; ++d)
#pragma unroll
            for (int e = 0; e < 16; ++e) {
                const int v = v0 + d * 32 + (e / 4) * 8 + lg * 4 + (e % 4);
                if (v < a.Dv) col[(size_t)v * a.R] = acc[d][e];
            }
    }
    if (threadIdx.x == 0 && blockIdx.x == 0) a.prod[(size_t)item * a.H + h] = expf((float)last);
}

// the state before every chunk of a request, in place of the chunk's own sum, and the request's new state
__global__ __launch_bounds__(256) void k_ssd_carry(SsdArgs a, int per_head) {
    const int b = blockIdx.z, h = blockIdx.y, e = blockIdx.x * 256 + threadIdx.x;
    const int first = a.requests[2 * b], n = a.requests[2 * b + 1];
    if (e >= per_head || n <= 0) return;
    float* sp = a.state + ((size_t)a.slots[b] * a.H + h) * per_head + e;
    float* cp = a.scratch + ((size_t)first * a.H + h) * per_head + e;
    const float* pp = a.prod + (size_t)first * a.H + h;
    const size_t step = (size_t)a.H * per_head;
    float t = *sp;
    for (int c0 = 0; c0 < n; c0 += 8) {          // eight chunks' loads on their way before the first is used
        float own[8], p[8];
#pragma unroll
        for (int u = 0; u < 8; ++u) {
            own[u] = c0 + u < n ? cp[(c0 + u) * step] : 0.f;
            p[u] = c0 + u < n ? pp[(size_t)(c0 + u) * a.H] : 1.f;
        }
#pragma unroll
        for (int u = 0; u < 8; ++u) {
            if (c0 + u >= n) break;
            cp[(c0 + u) * step] = t;
            t = fmaf(p[u], t, own[u]);
        }
    }
    *sp = t;
}

// KN: steps of 16 state rows that a lane's operands hold
template <int KN>
__global__ __launch_bounds__(256) void k_ssd_out(SsdArgs a) {
    constexpr int BLD = KN * 16 + 8;
    extern __shared__ __attribute__((aligned(16))) bf16_t lds[];
    bf16_t* xt = lds;                                   // [SSD_V][SSD_LD]
    bf16_t* bs = xt + SSD_V * SSD_LD;                   // [SSD_L][BLD]
    __shared__ float dt[SSD_L];
    __shared__ double cum[SSD_L];
    const int item = blockIdx.z, h = blockIdx.y, v0 = blockIdx.x * SSD_V;
    const int row0 = a.items[item * 4 + 1], rows = a.items[item * 4 + 2];
    ssd_steps(a, h, row0, rows, dt, cum);
    const int g = h / (a.H / a.G);
    load_transposed(xt, (bf16_t*)nullptr, a.x + h * a.Dv + v0, a.ld, row0, rows, a.Dv - v0, SSD_V / 8, [](int, float v) { return v; });
    for (int q = threadIdx.x; q < SSD_L * KN * 2; q += 256) {
        const int j = q / (KN * 2), n = (q - j * (KN * 2)) * 8;
        uint4 w = make_uint4(0, 0, 0, 0);
        if (j < rows && n < a.N) w = *reinterpret_cast<const uint4*>(a.b + (size_t)(row0 + j) * a.ld + g * a.N + n);
        *reinterpret_cast<uint4*>(bs + j * BLD + n) = w;
    }
    __syncthreads();
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, lr = lane & 31, lg = lane >> 5;
    const int i = wave * 32 + lr;                       // this lane's row of the chunk
    if (wave * 32 >= rows) return;
    const bool row_ok = i < rows;
    uint4 cf[KN];
#pragma unroll
    for (int ks = 0; ks < KN; ++ks) {
        const int n = ks * 16 + lg * 8;
        cf[ks] = make_uint4(0, 0, 0, 0);
        if (row_ok && n < a.N) cf[ks] = *reinterpret_cast<const uint4*>(a.c + (size_t)(row0 + i) * a.ld + g * a.N + n);
    }
    const int J = (a.N + a.R - 1) / a.R;
    const float* cp = a.scratch + ((size_t)item * a.H + h) * J * a.Dv * a.R;
    sd_f32x16 o[2];
#pragma unroll
    for (int d = 0; d < 2; ++d)
#pragma unroll
        for (int e = 0; e < 16; ++e) o[d][e] = 0.f;
    // what the state before the chunk gives: O^T[v, i] = S^T[v, n] C^T[n, i]
#pragma unroll
    for (int ks = 0; ks < KN; ++ks) {
        const int n = ks * 16 + lg * 8;
        if (ks * 16 >= a.N) break;
#pragma unroll
        for (int d = 0; d < 2; ++d) {
            const int v = v0 + d * 32 + lr;
            float4 s0 = make_float4(0.f, 0.f, 0.f, 0.f), s1 = s0;
            if (v < a.Dv && n < a.N) {       // (8 rows from a multiple of 8, in fours that lie side by side for both R)
                s0 = *reinterpret_cast<const float4*>(cp + ((size_t)(n / a.R) * a.Dv + v) * a.R + n % a.R);
                s1 = *reinterpret_cast<const float4*>(cp + ((size_t)((n + 4) / a.R) * a.Dv + v) * a.R + (n + 4) % a.R);
            }
            uint4 hi, lo;
            split2(s0.x, s0.y, hi.x, lo.x); split2(s0.z, s0.w, hi.y, lo.y);
            split2(s1.x, s1.y, hi.z, lo.z); split2(s1.z, s1.w, hi.w, lo.w);
            o[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(sd_frag(hi), sd_frag(cf[ks]), o[d], 0, 0, 0);
            o[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(sd_frag(lo), sd_frag(cf[ks]), o[d], 0, 0, 0);
        }
    }
    const double ci = cum[i];
    const float lead = expf((float)ci);
#pragma unroll
    for (int d = 0; d < 2; ++d)
#pragma unroll
        for (int e = 0; e < 16; ++e) o[d][e] *= lead;
    // what the chunk's own rows give
    const int ra = lr >> 3, rg = (lr >> 2) & 1, rb = lr & 3;
    const int key_off = 16 * (ra >> 1) + 8 * rg + 4 * (ra & 1) + rb;
    for (int jt = 0; jt <= wave; ++jt) {
        sd_f32x16 s;
#pragma unroll
        for (int e = 0; e < 16; ++e) s[e] = 0.f;
#pragma unroll
        for (int ks = 0; ks < KN; ++ks)
            s = __builtin_amdgcn_mfma_f32_32x32x16_bf16(sd_frag(*reinterpret_cast<const uint4*>(bs + (jt * 32 + key_off) * BLD + ks * 16 + lg * 8)),
                                                        sd_frag(cf[ks]), s, 0, 0, 0);
        float w[16];
#pragma unroll
        for (int e = 0; e < 16; ++e) {
            const int j = jt * 32 + 16 * (e >> 3) + 8 * lg + (e & 7);
            w[e] = j <= i ? s[e] * (dt[j] * expf((float)(ci - cum[j]))) : 0.f;
        }
#pragma unroll
        for (int jj = 0; jj < 2; ++jj) {
            uint4 hi, lo;
            split2(w[8 * jj], w[8 * jj + 1], hi.x, lo.x); split2(w[8 * jj + 2], w[8 * jj + 3], hi.y, lo.y);
            split2(w[8 * jj + 4], w[8 * jj + 5], hi.z, lo.z); split2(w[8 * jj + 6], w[8 * jj + 7], hi.w, lo.w);
#pragma unroll
            for (int d = 0; d < 2; ++d) {
                const sd_bf16x8 xf = sd_frag(*reinterpret_cast<const uint4*>(xt + (d * 32 + lr) * SSD_LD + jt * 32 + 16 * jj + 8 * lg));
                o[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(xf, sd_frag(hi), o[d], 0, 0, 0);
                o[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(xf, sd_frag(lo), o[d], 0, 0, 0);
            }
        }
    }
    if (!row_ok) return;
    const float skip = a.constants[2 * a.H + h];
    float* orow = a.out + (size_t)(row0 + i) * a.H * a.Dv + (size_t)h * a.Dv;
    const bf16_t* xrow = a.x + (size_t)(row0 + i) * a.ld + (size_t)h * a.Dv;
#pragma unroll
    for (int d = 0; d < 2; ++d)
#pragma unroll
        for (int e4 = 0; e4 < 4; ++e4) {
            const int v = v0 + d * 32 + e4 * 8 + lg * 4;
            if (v >= a.Dv) continue;             // (a multiple of 8: all four channels exist)
            const uint2 x = *reinterpret_cast<const uint2*>(xrow + v);
            *reinterpret_cast<float4*>(orow + v) = make_float4(
                fmaf(skip, __uint_as_float(x.x << 16), o[d][e4 * 4 + 0]), fmaf(skip, __uint_as_float(x.x & 0xffff0000u), o[d][e4 * 4 + 1]),
                fmaf(skip, __uint_as_float(x.y << 16), o[d][e4 * 4 + 2]), fmaf(skip, __uint_as_float(x.y & 0xffff0000u), o[d][e4 * 4 + 3]));
        }
}

extern "C" int xr_ssd_chunk_rows() { return SSD_L; }

template <typename K>
static int ssd_lds(K kernel, int bytes, bool& done) {
    if (done) return XR_OK;
    const hipError_t e = hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, bytes);
    if (e != hipSuccess) (void)hipGetLastError();     // or the next launch's check would report this refusal
    XR_REQUIRE(e == hipSuccess, "ssd: %d bytes of LDS refused: %s", bytes, hipGetErrorString(e));
    done = true;
    return XR_OK;
}

template <int NB>
static int launch_ssd(const SsdArgs& a, int n_items, int B, hipStream_t stream) {
    static bool state_ready = false, out_ready = false;
    constexpr int state_bytes = (2 * SSD_V + 32 * NB) * SSD_LD * 2, out_bytes = (SSD_V * SSD_LD + SSD_L * (NB * 32 + 8)) * 2;
    static_assert(state_bytes + SSD_L * 12 <= 160 * 1024 && out_bytes + SSD_L * 12 <= 160 * 1024, "the chunk does not fit into LDS");
    int rc = ssd_lds(k_ssd_state<NB>, state_bytes, state_ready);
    if (rc == XR_OK) rc = ssd_lds(k_ssd_out<2 * NB>, out_bytes, out_ready);
    if (rc != XR_OK) return rc;
    const dim3 grid((a.Dv + SSD_V - 1) / SSD_V, a.H, n_items);
    k_ssd_state<NB><<<grid, 256, state_bytes, stream>>>(a);
    XR_CHECK_LAUNCH("ssd_state");
    const int per_head = (a.N + a.R - 1) / a.R * a.Dv * a.R;
    k_ssd_carry<<<dim3((per_head + 255) / 256, a.H, B), 256, 0, stream>>>(a, per_head);
    XR_CHECK_LAUNCH("ssd_carry");
    k_ssd_out<2 * NB><<<grid, 256, out_bytes, stream>>>(a);
    XR_CHECK_LAUNCH("ssd_out");
    return XR_OK;
}

extern "C" int xr_ssd_chunks(float* out, const void* x, const void* b, const void* c, const float* z, const float* constants,
                             float* state, float* scratch, float* prod, const int* items, int n_items, const int* requests,
                             const int* slots, int B, int H, int G, int N, int Dv, int R, int ld, int ld_z, hipStream_t stream) {
    XR_REQUIRE(B >= 0 && n_items >= 0 && H > 0 && G > 0 && H % G == 0, "ssd: %d heads over %d groups", H, G);
    XR_REQUIRE(N > 0 && N <= 256 && N % 8 == 0 && Dv > 0 && Dv % 8 == 0, "ssd: states of %d (a multiple of 8 up to 256), values of %d (a multiple of 8)", N, Dv);
    XR_REQUIRE(R == 4 || R == 16, "ssd: state rows in groups of %d", R);
    XR_REQUIRE(ld % 8 == 0 && ld_z >= H && ((uintptr_t)x % 16) == 0 && ((uintptr_t)b % 16) == 0 && ((uintptr_t)c % 16) == 0,
               "ssd: rows of x, B and C must begin on 16 bytes (%d apart)", ld);
    XR_REQUIRE(((uintptr_t)out % 16) == 0 && ((uintptr_t)scratch % 16) == 0, "ssd: output and scratch must be 16-byte aligned");
    XR_REQUIRE(out && x && b && c && z && constants && state && scratch && prod && items && requests && slots, "ssd: a pointer is missing");
    XR_REQUIRE(n_items <= 65535 && B <= 65535, "ssd: %d chunks of %d requests", n_items, B);
    if (B == 0 || n_items == 0) return XR_OK;
    SsdArgs a{out, (const bf16_t*)x, (const bf16_t*)b, (const bf16_t*)c, z, constants, state, scratch, prod, items, requests, slots, H, G, N, Dv, R, ld, ld_z};
    if (N <= 64) return launch_ssd<2>(a, n_items, B, stream);
    if (N <= 128) return launch_ssd<4>(a, n_items, B, stream);
    return launch_ssd<8>(a, n_items, B, stream);
}
