// Sequence-mixing kernels for hybrid models (gfx950): LayerNorm and RMS norms on
// an fp32 residual stream (with the post-norm residual step fused),
// short causal convolutions with a carried tail, paged KV scatter with distinct
// K/V head sizes, interleaved rotary positions, paged softmax attention with
// optional sliding window / always-visible first tokens / log-distance penalty /
// query temperature / tanh score cap / softmax sink, linear recurrences with matrix
// state (gated delta rule, decayed scans, chunked gated linear attention, matrix memory
// with exponential gates), parallel residual streams, routers, and gated feed-forward
// activations.
//
// Built as a plain C-ABI shared library (no torch headers): the Python side
// passes raw device pointers and the current HIP stream, so the kernels are
// stream-ordered with the surrounding torch ops and hipGraph-capturable.
//
// Step layout shared by all kernels: activations are (B, S, ...) row-major;
// `pos` (B,S) int32 holds each token's position or -1 for padding; the real
// tokens of a row sit at columns 0..n-1 with consecutive positions; `seq`
// (B) int32 is the row's state slot or -1; `nvalid` (B) int32 is n.
// Statistics, scores, softmax, decays and the recurrent state are fp32
// regardless of the activation type.

#include <hip/hip_runtime.h>
#include <hip/hip_bf16.h>
#include <stdint.h>

#define WAVE 64
#define DEV __device__ __forceinline__

typedef __hip_bfloat16 bf16;

template <typename T> DEV float ldf(const T* p);
template <> DEV float ldf<float>(const float* p) { return *p; }
template <> DEV float ldf<bf16>(const bf16* p) { return __bfloat162float(*p); }
template <typename T> DEV void stf(T* p, float v);
template <> DEV void stf<float>(float* p, float v) { *p = v; }
template <> DEV void stf<bf16>(bf16* p, float v) { *p = __float2bfloat16(v); }

DEV float wave_sum(float v) {
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o, WAVE);
    return v;
}
DEV float wave_max(float v) {
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) v = fmaxf(v, __shfl_xor(v, o, WAVE));
    return v;
}
DEV float sigmoidf_(float x) { return 1.f / (1.f + expf(-x)); }
DEV float softplusf_(float x) { return x > 20.f ? x : log1pf(expf(x)); }

// 8 consecutive elements as floats, one or two 16-byte loads
template <typename T> DEV void load8(const T* p, float* v);
template <> DEV void load8<bf16>(const bf16* p, float* v) {
    const uint4 raw = *reinterpret_cast<const uint4*>(p);
    const uint32_t u[4] = {raw.x, raw.y, raw.z, raw.w};
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        v[2 * e] = __uint_as_float(u[e] << 16);
        v[2 * e + 1] = __uint_as_float(u[e] & 0xffff0000u);
    }
}
template <> DEV void load8<float>(const float* p, float* v) {
    const float4 a = *reinterpret_cast<const float4*>(p);
    const float4 b = *reinterpret_cast<const float4*>(p + 4);
    v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w;
    v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
}


// ---------------------------------------------------------------- LayerNorm
// one 256-thread workgroup per row; mean, then variance of the deviations
// (both fp32); the row is re-read from cache, not kept in registers, so any
// width works
#define LN_THREADS 256

DEV float block_sum(float v, float* red) {
    v = wave_sum(v);
    const int lane = threadIdx.x & (WAVE - 1), wv = threadIdx.x / WAVE;
    __syncthreads();                       // red may still be read by the previous call
    if (lane == 0) red[wv] = v;
    __syncthreads();
    float t = 0.f;
#pragma unroll
    for (int i = 0; i < LN_THREADS / WAVE; ++i) t += red[i];
    return t;
}

template <typename TOut>
__global__ void __launch_bounds__(LN_THREADS)
layer_norm_kernel(const float* __restrict__ x, const float* __restrict__ w,
                  const float* __restrict__ bias, TOut* __restrict__ out, long rows, int C,
                  float eps) {
    __shared__ float red[LN_THREADS / WAVE];
    const long row = blockIdx.x;
    const float* xr = x + row * C;
    float s = 0.f;
    for (int c = threadIdx.x; c < C; c += LN_THREADS) s += xr[c];
    const float mean = block_sum(s, red) / C;
    float v = 0.f;
    for (int c = threadIdx.x; c < C; c += LN_THREADS) { float d = xr[c] - mean; v += d * d; }
    const float inv = 1.f / sqrtf(block_sum(v, red) / C + eps);
    TOut* o = out + row * C;
    for (int c = threadIdx.x; c < C; c += LN_THREADS)
        stf<TOut>(o + c, (xr[c] - mean) * inv * w[c] + (bias ? bias[c] : 0.f));
}

// ------------------------------------------------------------- short conv
// y[b,t,c] = act(sum_j w[c,j] * x[b, t-R+j, c]) (+ x[b,t,c]); columns before
// the step come from the carried tail (oldest first), positions < 0 are zero
// y[b,t,c] = act(sum_j w[c,j] * x[b, t-R+j, c]) (+ x[b,t,c]); columns before
// the step come from the carried tail (oldest first), positions < 0 are zero.
// `xs` is the input's row stride in elements (a column slice of a wider
// projection is read in place); y is dense. One thread per element: adjacent
// lanes read adjacent channels of the same row for every tap.
template <typename TIn, typename TOut>
__global__ void short_conv_kernel(const TIn* __restrict__ x, long xs, const float* __restrict__ w,
                                  const float* __restrict__ tail, const int* __restrict__ pos,
                                  const int* __restrict__ seq, TOut* __restrict__ y,
                                  int B, int S, int C, int taps, int act_silu, int residual,
                                  const float* __restrict__ bias) {
    const long total = (long)B * S * C;
    const int R = taps - 1;
    for (long idx = (long)blockIdx.x * blockDim.x + threadIdx.x; idx < total;
         idx += (long)gridDim.x * blockDim.x) {
        const int c = idx % C;
        const long bt = idx / C;
        const int t = bt % S;
        const int b = bt / S;
        const int p = pos[bt];
        const int slot = seq[b];
        if (p < 0 || slot < 0) { stf<TOut>(y + idx, 0.f); continue; }
        const float* wr = w + (long)c * taps;
        float acc = bias ? bias[c] : 0.f, cur = 0.f;
        for (int j = 0; j < taps; ++j) {
            const int col = t - R + j;
            float xv;
            if (col >= 0) {
                xv = ldf<TIn>(x + ((long)b * S + col) * xs + c);
            } else {
                const int ps = p - R + j;              // source position
                xv = ps < 0 ? 0.f : tail[((long)slot * R + (R + col)) * C + c];
            }
            acc += wr[j] * xv;
            cur = xv;
        }
        if (act_silu) acc = acc * sigmoidf_(acc);
        if (residual) acc += cur;
        stf<TOut>(y + idx, acc);
    }
}

// Tiled variant for the common filter lengths: a thread owns 8 adjacent
// channels, keeps their taps in registers and walks SC_TT consecutive tokens
// with a sliding window of the last TAPS-1 inputs, so every input element is
// loaded once (16 bytes per load) instead of TAPS times.
#define SC_TT 16

template <typename T> DEV void st8(T* p, const float* v);
template <> DEV void st8<float>(float* p, const float* v) {
    *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
    *reinterpret_cast<float4*>(p + 4) = make_float4(v[4], v[5], v[6], v[7]);
}

template <typename TIn, typename TOut, int TAPS>
__global__ void short_conv_tile_kernel(const TIn* __restrict__ x, long xs,
                                       const float* __restrict__ w,
                                       const float* __restrict__ tail,
                                       const int* __restrict__ pos, const int* __restrict__ seq,
                                       const int* __restrict__ nvalid, TOut* __restrict__ y,
                                       int S, int C, int tiles_per_row, int act_silu,
                                       int residual, const float* __restrict__ bias) {
    constexpr int R = TAPS - 1;
    const int c = (blockIdx.x * blockDim.x + threadIdx.x) * 8;
    if (c >= C) return;
    const int b = blockIdx.y / tiles_per_row;
    const int t0 = (blockIdx.y % tiles_per_row) * SC_TT;
    const int t1 = min(t0 + SC_TT, S);
    const int slot = seq[b];
    const int n = slot < 0 ? 0 : nvalid[b];
    const int p0 = pos[(long)b * S];
    float wr[8][TAPS];
#pragma unroll
    for (int e = 0; e < 8; ++e)
#pragma unroll
        for (int j = 0; j < TAPS; ++j) wr[e][j] = w[(long)(c + e) * TAPS + j];
    float bs[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) bs[e] = bias ? bias[c + e] : 0.f;
    float hist[R > 0 ? R : 1][8];
#pragma unroll
    for (int r = 0; r < R; ++r) {
        const int col = t0 - R + r;
        if (col >= 0) {
            load8<TIn>(x + ((long)b * S + col) * xs + c, hist[r]);
        } else {
            const float* tp = tail + ((long)(slot < 0 ? 0 : slot) * R + (R + col)) * C + c;
#pragma unroll
            for (int e = 0; e < 8; ++e) hist[r][e] = (n > 0 && p0 + col >= 0) ? tp[e] : 0.f;
        }
    }
    for (int t = t0; t < t1; ++t) {
        float o[8];
        if (t < n) {
            float cur[8];
            load8<TIn>(x + ((long)b * S + t) * xs + c, cur);
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                float acc = bs[e];
#pragma unroll
                for (int r = 0; r < R; ++r) acc += wr[e][r] * hist[r][e];
                acc += wr[e][R] * cur[e];
                if (act_silu) acc = acc * sigmoidf_(acc);
                if (residual) acc += cur[e];
                o[e] = acc;
            }
#pragma unroll
            for (int r = 0; r + 1 < R; ++r)
#pragma unroll
                for (int e = 0; e < 8; ++e) hist[r][e] = hist[r + 1][e];
            if (R > 0) {
#pragma unroll
                for (int e = 0; e < 8; ++e) hist[R - 1][e] = cur[e];
            }
        } else {
#pragma unroll
            for (int e = 0; e < 8; ++e) o[e] = 0.f;
        }
        TOut* yp = y + ((long)b * S + t) * C + c;
        if constexpr (sizeof(TOut) == 2) {
            uint32_t pk[4];
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                uint32_t lo = __float_as_uint(o[2 * e]), hi = __float_as_uint(o[2 * e + 1]);
                lo += 0x7fffu + ((lo >> 16) & 1u);
                hi += 0x7fffu + ((hi >> 16) & 1u);
                pk[e] = (lo >> 16) | (hi & 0xffff0000u);
            }
            *reinterpret_cast<uint4*>(yp) = make_uint4(pk[0], pk[1], pk[2], pk[3]);
        } else {
            st8<float>(reinterpret_cast<float*>(yp), o);
        }
    }
}

// new tail = last R inputs of (old tail ++ this step's inputs); one thread per
// (row, channel) so the in-place shift is private to the thread
template <typename TIn>
__global__ void short_conv_commit_kernel(const TIn* __restrict__ x, long xs,
                                         float* __restrict__ tail,
                                         const int* __restrict__ pos, const int* __restrict__ seq,
                                         const int* __restrict__ nvalid, int B, int S, int C, int R) {
    const long idx = (long)blockIdx.x * blockDim.x + threadIdx.x;
    if (idx >= (long)B * C) return;
    const int c = idx % C;
    const int b = idx / C;
    const int slot = seq[b];
    const int n = nvalid[b];
    if (slot < 0 || n <= 0) return;
    const int p0 = pos[(long)b * S];
    float* tr = tail + (long)slot * R * C + c;
    for (int r = 0; r < R; ++r) {
        const int col = n - R + r;
        float v;
        if (col >= 0) v = ldf<TIn>(x + ((long)b * S + col) * xs + c);
        else v = (p0 + col) < 0 ? 0.f : tr[(long)(R + col) * C];
        tr[(long)r * C] = v;
    }
}

// ------------------------------------------------------------ paged KV write
template <typename T>
__global__ void paged_kv_write_kernel(T* __restrict__ kc, T* __restrict__ vc,
                                      const T* __restrict__ k, long kstride,
                                      const T* __restrict__ v, long vstride,
                                      const int* __restrict__ slots, long N, int GDk, int GDv,
                                      long nslots) {
    const int per = GDk + GDv;
    const long total = N * per;
    for (long idx = (long)blockIdx.x * blockDim.x + threadIdx.x; idx < total;
         idx += (long)gridDim.x * blockDim.x) {
        const long tok = idx / per;
        const int e = idx % per;
        const int s = slots[tok];
        if (s < 0 || s >= nslots) continue;
        if (e < GDk) kc[(long)s * GDk + e] = k[tok * kstride + e];
        else vc[(long)s * GDv + (e - GDk)] = v[tok * vstride + (e - GDk)];   // GDv = 0: no V
    }
}

// --------------------------------------------- latent cache row, one launch
// A latent layer's cache row of a token: [rms_norm(x[:C]) * w | x[C:C+R] with its
// first 2*half channels turned in interleaved (split = 0: 2i, 2i+1) or half-split
// (split = 1: i, i+half) pairs by pos * inv_freq[i]], written straight into the token's page slot (and, when `row` is given, into a dense row
// buffer as well). One wave per token; statistics and angles in fp32. Pad tokens
// (slot or position < 0) write nothing to the cache.
template <typename T>
__global__ void latent_row_kernel(const T* __restrict__ x, long xs, const float* __restrict__ w,
                                  float eps, const float* __restrict__ inv_freq, int half,
                                  int split,
                                  const int* __restrict__ pos, const int* __restrict__ slots,
                                  T* __restrict__ cache, long nslots, T* __restrict__ row, long rs,
                                  long ntok, int C, int R) {
    const int lane = threadIdx.x & (WAVE - 1);
    const long tok = (long)blockIdx.x * (blockDim.x / WAVE) + threadIdx.x / WAVE;
    if (tok >= ntok) return;
    const int s = slots[tok], p = pos[tok];
    T* cp = (s >= 0 && s < nslots && p >= 0) ? cache + (long)s * (C + R) : nullptr;
    T* rp = row ? row + tok * rs : nullptr;
    if (!cp && !rp) return;
    const T* xr = x + tok * xs;
    float ss = 0.f;
    for (int c = lane; c < C; c += WAVE) { const float v = ldf<T>(xr + c); ss += v * v; }
    const float inv = 1.f / sqrtf(wave_sum(ss) / C + eps);
    for (int c = lane; c < C; c += WAVE) {
        const float v = ldf<T>(xr + c) * inv * w[c];
        if (cp) stf<T>(cp + c, v);
        if (rp) stf<T>(rp + c, v);
    }
    for (int e = lane; e < half + (R - 2 * half); e += WAVE) {
        if (e < half) {
            const int c0 = C + (split ? e : 2 * e), c1 = C + (split ? e + half : 2 * e + 1);
            const float a = ldf<T>(xr + c0), b = ldf<T>(xr + c1);
            float sn, cs;
            sincosf((float)(p < 0 ? 0 : p) * inv_freq[e], &sn, &cs);
            const float u = a * cs - b * sn, v = b * cs + a * sn;
            if (cp) { stf<T>(cp + c0, u); stf<T>(cp + c1, v); }
            if (rp) { stf<T>(rp + c0, u); stf<T>(rp + c1, v); }
        } else {
            const int c = C + 2 * half + (e - half);
            const float v = ldf<T>(xr + c);
            if (cp) stf<T>(cp + c, v);
            if (rp) stf<T>(rp + c, v);
        }
    }
}

// ----------------------------------------------------------- paged attention
// Score of query i and key j, in order: q.k * scale * temp(i), temp(i) = 1 +
// qt_coef * ln(floor((i+1)/qt_every) + 1) (qt_every = 0: none); minus
// r1_h * log(1 + r2_h (i-j)) (r1 = null: none); cap * tanh(. / cap) (cap = 0:
// none); a lone r1 (r2 = null) is a linear penalty r1_h * (i-j) instead.
// Visible: j <= i and (i-j < window or j < keep); plain causal attention
// passes window = INT_MAX. With cmask > 0 also only keys of the query's own block
// of cmask positions (j >= floor(i/cmask)*cmask). `sink` (per head, or null)
// adds exp(sink_h) to the softmax denominator. K and V rows are addressed as slot*tok_stride +
// head*head_stride, so V may be a channel range of the K rows.
// Workgroup (4 waves) = ATT_NQ query rows that share one KV head: HPW query
// heads of the group x QT consecutive tokens of a batch row, so every K/V
// line fetched serves all of them. The union of the rows' visible keys is
// [0, min(keep, lo)) + [lo, i_max], lo = the larger of max(0, i_min-window+1)
// and i_min's block start; each row masks by its own position. Waves
// take 64-key tiles round-robin: a lane owns one key for the scores (q rows
// broadcast from LDS, fp32 accumulate, online softmax per row), then the
// wave's P tile goes through LDS and a lane owns value channels for P.V.
// The four partial results merge through LDS at the end. One kernel serves
// prompt portions, decoded tokens and mixed batches.
// Two shapes: (NQ=16 rows, 4 waves) for steps with prompt portions, and
// (NQ=4 rows, 16 waves) for pure decode steps, where one token's few heads
// leave the key range as the only parallelism.
#define ATT_NQ_MAX 16

template <typename T, typename TOut, int MAXR, int ATT_NQ, int ATT_WAVES>
__global__ void __launch_bounds__(ATT_WAVES * WAVE)
window_attn_kernel(const T* __restrict__ q, long qstride, const T* __restrict__ kc,
                   const T* __restrict__ vc, const int* __restrict__ pos,
                   const int* __restrict__ seq,
                   const int* __restrict__ btab, int max_blocks, const float* __restrict__ r1,
                   const float* __restrict__ r2, const T* __restrict__ gate, long gstride,
                   TOut* __restrict__ out, int H, int G, int Dk, int Dv,
                   int bsz, int S, float scale, int window, int keep, int HPW, int QT,
                   int chunks, int lpr, int pws, long ktok, long khead, long vtok, long vhead,
                   int kvec, const float* __restrict__ sink, float cap, float qt_coef,
                   int qt_every, int ghead, int cmask) {
    // lpr > 0 (decode shape only): P.V with 8 value channels per lane and
    // 64/lpr keys per step, 16-byte V loads; pws = floats of LDS per wave
    extern __shared__ __attribute__((aligned(16))) float smem[];
    const int DkP = (Dk + 7) & ~7;                       // padded q row
    float* qs = smem;                                    // ATT_NQ * DkP
    float* ps = qs + ATT_NQ * DkP;                       // ATT_WAVES * 64 * ATT_NQ
    float* cs = ps;                                      // merge area reuses the P tiles
    constexpr int ATT_THREADS = ATT_WAVES * WAVE;
    __shared__ int rpos[ATT_NQ_MAX], rclo[ATT_NQ_MAX];
    __shared__ float ra1[ATT_NQ_MAX], ra2[ATT_NQ_MAX], rtemp[ATT_NQ_MAX], rsink[ATT_NQ_MAX];

    const int tid = threadIdx.x, lane = tid & (WAVE - 1), wv = tid / WAVE;
    const int b = blockIdx.z;
    const int g = blockIdx.y / chunks, chunk = blockIdx.y % chunks;
    const int t0 = blockIdx.x * QT;
    const int rep = H / G;
    if (seq[b] < 0) return;
    // row table
    if (tid < ATT_NQ) {
        const int tq = tid / HPW, hh = chunk * HPW + tid % HPW;
        int p = -1;
        if (tq < QT && t0 + tq < S && hh < rep) p = pos[(long)b * S + t0 + tq];
        rpos[tid] = p;
        rclo[tid] = (cmask > 0 && p >= 0) ? (p / cmask) * cmask : 0;
        const int h = g * rep + (hh < rep ? hh : 0);
        ra1[tid] = r1 ? r1[h] : 0.f;
        ra2[tid] = r2 ? r2[h] : 0.f;
        rsink[tid] = sink ? sink[h] : -INFINITY;
        rtemp[tid] = (qt_every > 0 && p >= 0)
            ? 1.f + qt_coef * logf((float)((p + 1) / qt_every) + 1.f) : 1.f;
    }
    __syncthreads();
    int i_min = 0x7fffffff, i_max = -1;
#pragma unroll
    for (int r = 0; r < ATT_NQ; ++r) {
        const int p = rpos[r];
        if (p >= 0) { i_min = min(i_min, p); i_max = max(i_max, p); }
    }
    if (i_max < 0) return;                               // uniform
    // q rows (scaled) into LDS
    for (int idx = tid; idx < ATT_NQ * DkP; idx += ATT_THREADS) {
        const int r = idx / DkP, d = idx % DkP;
        float v = 0.f;
        if (rpos[r] >= 0 && d < Dk) {
            const int tq = r / HPW, h = g * rep + chunk * HPW + r % HPW;
            v = ldf<T>(q + ((long)b * S + t0 + tq) * qstride + (long)h * Dk + d) * (scale * rtemp[r]);
        }
        qs[idx] = v;
    }
    __syncthreads();

    const int* bt = btab + (long)b * max_blocks;
    const int lo = max(max(0, i_min - window + 1), cmask > 0 ? (i_min / cmask) * cmask : 0);
    const int nfirst = min(keep, lo);
    const int n = nfirst + (i_max - lo + 1);
    const int ntiles = (n + WAVE - 1) / WAVE;
    const int rounds = (ntiles + ATT_WAVES - 1) / ATT_WAVES;
    float m_run[ATT_NQ], l_run[ATT_NQ], acc[ATT_NQ][MAXR];
#pragma unroll
    for (int r = 0; r < ATT_NQ; ++r) {
        m_run[r] = -INFINITY; l_run[r] = 0.f;
#pragma unroll
        for (int c = 0; c < MAXR; ++c) acc[r][c] = 0.f;
    }
    float* myp = ps + wv * pws;
    constexpr int NV = ATT_NQ == 4 ? 8 : 1;
    float acc8[ATT_NQ == 4 ? 4 : 1][NV];
#pragma unroll
    for (int r = 0; r < (ATT_NQ == 4 ? 4 : 1); ++r)
#pragma unroll
        for (int e = 0; e < NV; ++e) acc8[r][e] = 0.f;

    for (int rd = 0; rd < rounds; ++rd) {
        const int base = (rd * ATT_WAVES + wv) * WAVE;
        const int m = base + lane;
        const bool kvalid = m < n;
        int j = 0;
        long slot = 0;
        float sc[ATT_NQ];
#pragma unroll
        for (int r = 0; r < ATT_NQ; ++r) sc[r] = 0.f;
        if (base < n) {                                  // wave-uniform
            if (kvalid) {
                j = m < nfirst ? m : lo + (m - nfirst);
                const int blk = bt[j / bsz];
                slot = (long)(blk < 0 ? 0 : blk) * bsz + (j % bsz);
            }
            const T* kp = kc + slot * ktok + (long)g * khead;
            if (kvec) {
                for (int d = 0; d < Dk; d += 8) {
                    float kv[8];
                    load8<T>(kp + d, kv);
#pragma unroll
                    for (int r = 0; r < ATT_NQ; ++r) {
                        if (rpos[r] < 0) continue;       // uniform
                        const float4 qa = *reinterpret_cast<const float4*>(qs + r * DkP + d);
                        const float4 qb = *reinterpret_cast<const float4*>(qs + r * DkP + d + 4);
                        sc[r] += kv[0] * qa.x + kv[1] * qa.y + kv[2] * qa.z + kv[3] * qa.w +
                                 kv[4] * qb.x + kv[5] * qb.y + kv[6] * qb.z + kv[7] * qb.w;
                    }
                }
            } else {
                for (int d = 0; d < Dk; ++d) {
                    const float kvs = ldf<T>(kp + d);
#pragma unroll
                    for (int r = 0; r < ATT_NQ; ++r) sc[r] += kvs * qs[r * DkP + d];
                }
            }
            // bias, mask, online softmax per row
#pragma unroll
            for (int r = 0; r < ATT_NQ; ++r) {
                const int i = rpos[r];
                if (i < 0) continue;                     // uniform
                const int dist = i - j;
                const bool vis = kvalid && dist >= 0 && (dist < window || j < keep) &&
                                 j >= rclo[r];
                float sv = -INFINITY;
                if (vis) {
                    sv = sc[r];
                    if (r1 && r2) {                      // uniform
                        const float x = ra2[r] * (float)dist;
                        const float lg = sizeof(T) == 4 ? log1pf(x) : __logf(1.f + x);
                        sv -= ra1[r] * lg;
                    } else if (r1) {
                        sv -= ra1[r] * (float)dist;
                    }
                    if (cap > 0.f) sv = cap * tanhf(sv / cap);
                }
                const float m_new = fmaxf(m_run[r], wave_max(sv));
                float p = 0.f, corr = 1.f;
                if (m_new > -INFINITY) {
                    p = vis ? expf(sv - m_new) : 0.f;
                    corr = expf(m_run[r] - m_new);
                }
                l_run[r] = l_run[r] * corr + wave_sum(p);
                m_run[r] = m_new;
#pragma unroll
                for (int c = 0; c < MAXR; ++c) acc[r][c] *= corr;
                if constexpr (ATT_NQ == 4) {
#pragma unroll
                    for (int e = 0; e < NV; ++e) acc8[r][e] *= corr;
                }
                sc[r] = p;
            }
#pragma unroll
            for (int r = 0; r < ATT_NQ; ++r) myp[lane * ATT_NQ + r] = sc[r];
        }
        __syncthreads();
        if (base < n) {
            const int cnt = min(WAVE, n - base);
            const int sl = (int)slot;
            bool done = false;
            if constexpr (ATT_NQ == 4) {
                if (lpr > 0) {
                    done = true;
                    const int ksub = WAVE / lpr;
                    const int sub = lane / lpr, ch = (lane % lpr) * 8;
                    for (int it = 0; it * ksub < cnt; ++it) {
                        const int mm = it * ksub + sub;
                        const long sj = __shfl(sl, mm < cnt ? mm : 0, WAVE);
                        if (mm < cnt) {
                            float vv[8];
                            load8<T>(vc + sj * vtok + (long)g * vhead + ch, vv);
                            const float4 pp = *reinterpret_cast<const float4*>(myp + mm * ATT_NQ);
#pragma unroll
                            for (int e = 0; e < 8; ++e) {
                                acc8[0][e] += pp.x * vv[e];
                                acc8[1][e] += pp.y * vv[e];
                                acc8[2][e] += pp.z * vv[e];
                                acc8[3][e] += pp.w * vv[e];
                            }
                        }
                    }
                }
            }
            if (!done) {
                for (int mm = 0; mm < cnt; ++mm) {
                    const long sj = __shfl(sl, mm, WAVE);
                    const T* vp = vc + sj * vtok + (long)g * vhead;
                    float vv[MAXR];
#pragma unroll
                    for (int c = 0; c < MAXR; ++c) {
                        const int d = lane + c * WAVE;
                        vv[c] = d < Dv ? ldf<T>(vp + d) : 0.f;
                    }
                    const float4* p4 = reinterpret_cast<const float4*>(myp + mm * ATT_NQ);
#pragma unroll
                    for (int r4 = 0; r4 < ATT_NQ / 4; ++r4) {
                        const float4 pp = p4[r4];
#pragma unroll
                        for (int c = 0; c < MAXR; ++c) {
                            acc[4 * r4][c] += pp.x * vv[c];
                            acc[4 * r4 + 1][c] += pp.y * vv[c];
                            acc[4 * r4 + 2][c] += pp.z * vv[c];
                            acc[4 * r4 + 3][c] += pp.w * vv[c];
                        }
                    }
                }
            }
        }
        __syncthreads();
    }
    if constexpr (ATT_NQ == 4) {
        if (lpr > 0) {
            // fold the key subgroups, then move to the channel-per-lane layout
            // the merge and the epilogue use (through this wave's LDS region)
#pragma unroll
            for (int r = 0; r < 4; ++r)
#pragma unroll
                for (int e = 0; e < 8; ++e) {
                    float v = acc8[r][e];
                    for (int off = lpr; off < WAVE; off <<= 1) v += __shfl_xor(v, off, WAVE);
                    if (lane < lpr) myp[r * Dv + lane * 8 + e] = v;
                }
            __syncthreads();
#pragma unroll
            for (int r = 0; r < 4; ++r)
#pragma unroll
                for (int c = 0; c < MAXR; ++c) {
                    const int d = lane + c * WAVE;
                    if (d < Dv) acc[r][c] = myp[r * Dv + d];
                }
            __syncthreads();
        }
    }
    // merge the waves' partial softmaxes pairwise (tree) through LDS
    for (int step = 1; step < ATT_WAVES; step <<= 1) {
        float* slot_acc = cs + (wv / (2 * step)) * ATT_NQ * (Dv + 2);
        float* cm = slot_acc + ATT_NQ * Dv;
        float* cl = cm + ATT_NQ;
        if (wv % (2 * step) == step) {
#pragma unroll
            for (int r = 0; r < ATT_NQ; ++r) {
                if (lane == 0) { cm[r] = m_run[r]; cl[r] = l_run[r]; }
#pragma unroll
                for (int c = 0; c < MAXR; ++c) {
                    const int d = lane + c * WAVE;
                    if (d < Dv) slot_acc[r * Dv + d] = acc[r][c];
                }
            }
        }
        __syncthreads();
        if (wv % (2 * step) == 0 && wv + step < ATT_WAVES) {
#pragma unroll
            for (int r = 0; r < ATT_NQ; ++r) {
                const float mo = cm[r], lo2 = cl[r];
                const float m_new = fmaxf(m_run[r], mo);
                float ca = 1.f, cb = 0.f;
                if (m_new > -INFINITY) { ca = expf(m_run[r] - m_new); cb = expf(mo - m_new); }
                l_run[r] = l_run[r] * ca + lo2 * cb;
                m_run[r] = m_new;
#pragma unroll
                for (int c = 0; c < MAXR; ++c) {
                    const int d = lane + c * WAVE;
                    if (d < Dv) acc[r][c] = acc[r][c] * ca + slot_acc[r * Dv + d] * cb;
                }
            }
        }
        __syncthreads();
    }
    if (wv != 0) return;
#pragma unroll
    for (int r = 0; r < ATT_NQ; ++r) {
        if (rpos[r] < 0) continue;
        const int tq = r / HPW, h = g * rep + chunk * HPW + r % HPW;
        const long tok = (long)b * S + t0 + tq;
        float inv = 1.f / l_run[r];
        if (sink) {                                      // one more term in the denominator
            const float mf = fmaxf(m_run[r], rsink[r]);
            const float ca = expf(m_run[r] - mf);
            inv = ca / (l_run[r] * ca + expf(rsink[r] - mf));
        }
        TOut* op = out + (tok * H + h) * (long)Dv;
        // gate: one number per value channel, or (ghead) one per head
        const T* gp = gate ? gate + tok * gstride + (ghead ? (long)h : (long)h * Dv) : nullptr;
        if (gp && ghead) inv *= sigmoidf_(ldf<T>(gp));
        if (ghead) gp = nullptr;
#pragma unroll
        for (int c = 0; c < MAXR; ++c) {
            const int d = lane + c * WAVE;
            if (d < Dv) {
                float o = acc[r][c] * inv;
                if (gp) o *= sigmoidf_(ldf<T>(gp + d));
                stf<TOut>(op + d, o);
            }
        }
    }
}

// -------------------------------------------------- paged attention, matrix cores
// bf16 prompt-portion path, same scores and options as above. Workgroup = 64
// query rows of one KV head (4 waves x 16 rows: the group's heads x consecutive
// tokens); all waves walk the same 64-key tiles, staged once in LDS (K row-major,
// V transposed). Scores are computed transposed, S^T = K Q^T (mfma 16x16x32 bf16,
// fp32 accumulate), so a lane ends up with 16 scores of ONE query row and the
// probabilities already sit in the A-operand layout of the P.V product. Scale,
// temperature, bias, cap, mask and online softmax are fp32 per lane; P enters the
// second product as a hi + lo bf16 pair (16 mantissa bits), V as stored.
// DKP / DVP are the head sizes padded to multiples of 32; the true Dk, Dv (any
// multiples of 8) come at run time and the padding is zero-filled in LDS. KT is
// the key tile (64, or 32 for wide keys so that the K tile still fits LDS). Values
// wider than DVP are split over `nsplit` workgroups that each recompute the scores
// and own DVP value channels (latent caches: a 576-wide key row whose first 512
// channels are the value).
typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
typedef float f32x4_t __attribute__((ext_vector_type(4)));
#define MA_ROWS 64

DEV uint16_t f2bf_rne(float f) {
    uint32_t u = __float_as_uint(f);
    u += 0x7fffu + ((u >> 16) & 1u);
    return (uint16_t)(u >> 16);
}

// bf16-only kernels take the hardware exponential: its 2^-21 relative error is
// far below the rounding of their operands
DEV float fast_tanh_(float y) { return 1.f - __fdividef(2.f, 1.f + __expf(2.f * y)); }

template <int DKP, int DVP, int MA_KT, bool PREFETCH>
__global__ void __launch_bounds__(256)
paged_attn_mfma_kernel(const bf16* __restrict__ q, long qstride, const bf16* __restrict__ kc,
                       const bf16* __restrict__ vc, const int* __restrict__ pos,
                       const int* __restrict__ seq, const int* __restrict__ btab,
                       int max_blocks, const float* __restrict__ r1,
                       const float* __restrict__ r2, const bf16* __restrict__ gate,
                       long gstride, bf16* __restrict__ out, int H, int G, int Dk, int Dv,
                       int bsz, int S, float scale, int window, int keep, int QT, long ktok,
                       long khead, long vtok, long vhead, const float* __restrict__ sink,
                       float cap, float qt_coef, int qt_every, int nsplit, int ghead,
                       int cmask) {
    constexpr int KB = MA_KT / 16;           // 16-key score blocks per tile
    constexpr int KS = DKP + 8;              // K tile row stride (elements)
    constexpr int VS = MA_KT + 8;            // V^T tile row stride
    __shared__ __attribute__((aligned(16))) uint16_t k_lds[MA_KT * KS];
    __shared__ __attribute__((aligned(16))) uint16_t vt_lds[DVP * VS];
    __shared__ int rpos[MA_ROWS];
    __shared__ float ra1[MA_ROWS], ra2[MA_ROWS], rsink[MA_ROWS];
    const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
    const int lr = lane & 15, lg = lane >> 4;
    // Workgroups go to the 8 XCDs in turn: renumber them so that an XCD works on
    // whole heads, whose keys and values then stay in its L2
    const int nwg = gridDim.x * gridDim.y;
    int wg = blockIdx.y * gridDim.x + blockIdx.x;
    if (nwg % 8 == 0) wg = (wg % 8) * (nwg / 8) + wg / 8;
    const int by = wg / gridDim.x, bx = wg % gridDim.x;
    // the last tokens of a row see the most keys: they start first
    const int b = blockIdx.z, g = by / nsplit, t0 = (gridDim.x - 1 - bx) * QT;
    const int dv0 = (by % nsplit) * DVP;         // first value channel of this split
    const int dvn = min(DVP, Dv - dv0);
    const int rep = H / G;
    if (seq[b] < 0) return;
    if (tid < MA_ROWS) {
        const int tq = tid / rep, hh = tid % rep;
        rpos[tid] = (tq < QT && t0 + tq < S) ? pos[(long)b * S + t0 + tq] : -1;
        ra1[tid] = r1 ? r1[g * rep + hh] : 0.f;
        ra2[tid] = r2 ? r2[g * rep + hh] : 0.f;
        rsink[tid] = sink ? sink[g * rep + hh] : -INFINITY;
    }
    __syncthreads();
    int i_min = 0x7fffffff, i_max = -1;
    for (int r = 0; r < MA_ROWS; r += rep) {     // one entry per token
        const int p = rpos[r];
        if (p >= 0) { i_min = min(i_min, p); i_max = max(i_max, p); }
    }
    if (i_max < 0) return;                       // uniform
    // this lane's query row (B operand of S^T): row = 16*wv + lr
    const int myrow = wv * 16 + lr;
    const int my_i = rpos[myrow];
    const int my_clo = (cmask > 0 && my_i >= 0) ? (my_i / cmask) * cmask : 0;
    const float a1 = ra1[myrow], a2 = ra2[myrow];
    const float qscale = (qt_every > 0 && my_i >= 0)
        ? scale * (1.f + qt_coef * logf((float)((my_i + 1) / qt_every) + 1.f)) : scale;
    bf16x8_t qf[DKP / 32];
    {
        const int tq = myrow / rep, h = g * rep + myrow % rep;
        const bf16* qp = q + ((long)b * S + t0 + tq) * qstride + (long)h * Dk;
#pragma unroll
        for (int ks = 0; ks < DKP / 32; ++ks) {
            uint4 raw = make_uint4(0, 0, 0, 0);
            if (my_i >= 0 && ks * 32 + lg * 8 < Dk)
                raw = *reinterpret_cast<const uint4*>(qp + ks * 32 + lg * 8);
            qf[ks] = *reinterpret_cast<bf16x8_t*>(&raw);
        }
    }
    const int* bt = btab + (long)b * max_blocks;
    const int lo = max(max(0, i_min - window + 1), cmask > 0 ? (i_min / cmask) * cmask : 0);
    const int clo_max = cmask > 0 ? (i_max / cmask) * cmask : 0;   // block start of the last row
    const int nfirst = min(keep, lo);
    const int n = nfirst + (i_max - lo + 1);
    float m_run = -INFINITY, l_run = 0.f;
    f32x4_t o_acc[DVP / 16];
#pragma unroll
    for (int nb = 0; nb < DVP / 16; ++nb) o_acc[nb] = f32x4_t{0.f, 0.f, 0.f, 0.f};

    // A tile's K and V lines travel global -> registers -> LDS, all loads of a tile in
    // flight together: the keys' cache slots are looked up one tile ahead (LDS, two
    // buffers) and addresses are clamped rather than branched around. With PREFETCH
    // the next tile's loads are issued before the current tile's products; without,
    // the registers are reused and more workgroups share a CU.
    __shared__ int kslot[2][MA_KT];
#define MA_SLOTS(BASE, BUF)                                                                \
    if (tid < MA_KT) {                                                                     \
        const int mm = min((BASE) + tid, n - 1);                                           \
        const int j = mm < nfirst ? mm : lo + (mm - nfirst);                               \
        const int blk = bt[j / bsz];                                                       \
        kslot[BUF][tid] = (blk < 0 ? 0 : blk) * bsz + (j % bsz);                           \
    }
    constexpr int NKI = (MA_KT * (DKP / 8) + 255) / 256;
    constexpr int NVI = (MA_KT * (DVP / 8) + 255) / 256;
    const bf16* kbase = kc + (long)g * khead;
    const bf16* vbase = vc + (long)g * vhead + dv0;
    uint4 rk[NKI], rv[NVI];
#define MA_FETCH(BASE, BUF)                                                                \
    {                                                                                      \
        _Pragma("unroll") for (int x = 0; x < NKI; ++x) {                                  \
            const int c = tid + x * 256;                                                   \
            const int m = min(c / (DKP / 8), MA_KT - 1), part = c % (DKP / 8);             \
            rk[x] = *reinterpret_cast<const uint4*>(                                       \
                kbase + (long)kslot[BUF][m] * ktok + min(part * 8, Dk - 8));               \
        }                                                                                  \
        _Pragma("unroll") for (int x = 0; x < NVI; ++x) {                                  \
            const int c = tid + x * 256;                                                   \
            const int m = c % MA_KT, part = c / MA_KT;   /* consecutive lanes: consecutive keys */ \
            rv[x] = *reinterpret_cast<const uint4*>(                                       \
                vbase + (long)kslot[BUF][m] * vtok + min(part * 8, dvn - 8));              \
        }                                                                                  \
    }
    MA_SLOTS(0, 0)
    __syncthreads();
    if constexpr (PREFETCH) MA_FETCH(0, 0)
    int buf = 0;
    for (int base = 0; base < n; base += MA_KT, buf ^= 1) {
        if constexpr (!PREFETCH) MA_FETCH(base, buf)
        if (base + MA_KT < n) MA_SLOTS(base + MA_KT, buf ^ 1)
        // ---- registers -> LDS: K row-major, V transposed; zeros past the last key
        // and the last channel
#pragma unroll
        for (int x = 0; x < NKI; ++x) {
            const int c = tid + x * 256;
            const int m = c / (DKP / 8), part = c % (DKP / 8);
            const bool ok = base + m < n && part * 8 < Dk;
            const uint4 raw = make_uint4(ok ? rk[x].x : 0, ok ? rk[x].y : 0, ok ? rk[x].z : 0,
                                         ok ? rk[x].w : 0);
            if (c < MA_KT * (DKP / 8))
                *reinterpret_cast<uint4*>(k_lds + m * KS + part * 8) = raw;
        }
#pragma unroll
        for (int x = 0; x < NVI; ++x) {
            const int c = tid + x * 256;
            const int m = c % MA_KT, part = c / MA_KT;
            const bool ok = base + m < n && part * 8 < dvn;
            const uint32_t u[4] = {ok ? rv[x].x : 0, ok ? rv[x].y : 0, ok ? rv[x].z : 0,
                                   ok ? rv[x].w : 0};
            if (c < MA_KT * (DVP / 8)) {
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    vt_lds[(part * 8 + 2 * e) * VS + m] = (uint16_t)(u[e] & 0xffffu);
                    vt_lds[(part * 8 + 2 * e + 1) * VS + m] = (uint16_t)(u[e] >> 16);
                }
            }
        }
        __syncthreads();
        if constexpr (PREFETCH) {
            if (base + MA_KT < n) MA_FETCH(base + MA_KT, buf ^ 1) // in flight during the products
        }
        // ---- S^T = K Q^T: lane gets keys 16*kb + 4*lg + r of its own row lr
        float sv[KB][4];
        float mt = -INFINITY;
        // a tile every row of the workgroup sees whole (all but the diagonal
        // tiles of a causal prompt) needs no per-score mask
        const bool whole = nfirst == 0 && base + MA_KT <= n && lo + base + MA_KT - 1 <= i_min &&
                           i_max - (lo + base) < window && lo + base >= clo_max;
#pragma unroll
        for (int kb = 0; kb < KB; ++kb) {
            f32x4_t acc = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int ks = 0; ks < DKP / 32; ++ks) {
                const bf16x8_t ka = *reinterpret_cast<const bf16x8_t*>(
                    k_lds + (kb * 16 + lr) * KS + ks * 32 + lg * 8);
                acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ka, qf[ks], acc, 0, 0, 0);
            }
            if (whole && !r2) {                          // uniform
                // (a linear penalty needs no mask either: the tile's keys are
                // lo + base + 16 kb + 4 lg + r, all at or before every row)
                const float d0 = (float)(my_i - (lo + base + kb * 16 + lg * 4));
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    float x = acc[r] * qscale;
                    if (r1) x -= a1 * (d0 - (float)r);
                    if (cap > 0.f) x = cap * fast_tanh_(x / cap);
                    if (my_i < 0) x = -INFINITY;
                    sv[kb][r] = x;
                    mt = fmaxf(mt, x);
                }
                continue;
            }
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int mm = base + kb * 16 + lg * 4 + r;
                const int j = mm < nfirst ? mm : lo + (mm - nfirst);
                const int dist = my_i - j;
                const bool vis = mm < n && my_i >= 0 && dist >= 0 && (dist < window || j < keep) &&
                                 j >= my_clo;
                float x = -INFINITY;
                if (vis) {
                    x = acc[r] * qscale;
                    if (r1) x -= r2 ? a1 * __logf(1.f + a2 * (float)dist) : a1 * (float)dist;
                    if (cap > 0.f) x = cap * fast_tanh_(x / cap);
                }
                sv[kb][r] = x;
                mt = fmaxf(mt, x);
            }
        }
        mt = fmaxf(mt, __shfl_xor(mt, 16, WAVE));
        mt = fmaxf(mt, __shfl_xor(mt, 32, WAVE));
        const float m_new = fmaxf(m_run, mt);
        float corr = 1.f, psum = 0.f;
        if (m_new > -INFINITY) {
            corr = __expf(m_run - m_new);
#pragma unroll
            for (int kb = 0; kb < KB; ++kb)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const float pv = sv[kb][r] > -INFINITY ? __expf(sv[kb][r] - m_new) : 0.f;
                    sv[kb][r] = pv;
                    psum += pv;
                }
        } else {
#pragma unroll
            for (int kb = 0; kb < KB; ++kb)
#pragma unroll
                for (int r = 0; r < 4; ++r) sv[kb][r] = 0.f;
        }
        psum += __shfl_xor(psum, 16, WAVE);
        psum += __shfl_xor(psum, 32, WAVE);
        l_run = l_run * corr + psum;
        m_run = m_new;
        // ---- rescale O: its rows are 4*lg + r, their corr sits in lane (4*lg + r)
        if (__any(corr != 1.f)) {                        // some row's maximum moved
            float cr[4];
#pragma unroll
            for (int r = 0; r < 4; ++r) cr[r] = __shfl(corr, lg * 4 + r, WAVE);
#pragma unroll
            for (int nb = 0; nb < DVP / 16; ++nb)
#pragma unroll
                for (int r = 0; r < 4; ++r) o_acc[nb][r] *= cr[r];
        }
        // ---- O += P V, 32 keys per product, P as hi + lo
#pragma unroll
        for (int kc2 = 0; kc2 < MA_KT / 32; ++kc2) {
            struct { bf16x8_t v; } ph, pl;               // hardware float -> bf16 (RNE)
#pragma unroll
            for (int jj = 0; jj < 8; ++jj) {
                const float pv = sv[2 * kc2 + (jj >> 2)][jj & 3];
                const __bf16 hb = (__bf16)pv;
                ph.v[jj] = hb;
                pl.v[jj] = (__bf16)(pv - (float)hb);
            }
#pragma unroll
            for (int nb = 0; nb < DVP / 16; ++nb) {
                union { bf16x8_t v; uint2 h[2]; } vb;
                const uint16_t* vp = vt_lds + (nb * 16 + lr) * VS + 32 * kc2 + 4 * lg;
                vb.h[0] = *reinterpret_cast<const uint2*>(vp);
                vb.h[1] = *reinterpret_cast<const uint2*>(vp + 16);
                o_acc[nb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ph.v, vb.v, o_acc[nb], 0, 0, 0);
                o_acc[nb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pl.v, vb.v, o_acc[nb], 0, 0, 0);
            }
        }
        __syncthreads();
    }
#undef MA_FETCH
#undef MA_SLOTS
    // ---- epilogue: rows 4*lg + r of this wave, channel 16*nb + lr. A sink adds
    // one term to the row's denominator (computed by the lane that owns the row)
    float fin = l_run > 0.f ? 1.f / l_run : 0.f;
    if (sink) {
        const float sk = rsink[myrow];
        const float mf = fmaxf(m_run, sk);
        const float ca = m_run > -INFINITY ? __expf(m_run - mf) : 0.f;
        fin = ca / (l_run * ca + __expf(sk - mf));
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        const int row = wv * 16 + lg * 4 + r;
        const float inv = __shfl(fin, lg * 4 + r, WAVE);
        if (rpos[row] < 0) continue;
        const int tq = row / rep, h = g * rep + row % rep;
        const long tok = (long)b * S + t0 + tq;
        bf16* op = out + (tok * H + h) * (long)Dv + dv0;
        const bf16* gp = (gate && !ghead) ? gate + tok * gstride + (long)h * Dv + dv0 : nullptr;
        const float hg = (gate && ghead)
            ? sigmoidf_(__bfloat162float(gate[tok * gstride + h])) : 1.f;
#pragma unroll
        for (int nb = 0; nb < DVP / 16; ++nb) {
            const int d = nb * 16 + lr;
            if (d >= dvn) continue;
            float o = o_acc[nb][r] * inv * hg;
            if (gp) o *= sigmoidf_(__bfloat162float(gp[d]));
            op[d] = __float2bfloat16(o);
        }
    }
}

// ------------------------------------ latent-cache decode, matrix cores
// Single-token steps of multi-query layers whose values are the first Dv
// channels of the (one) key row per token — the absorbed form of latent
// attention: 16 query heads of one token are the 16 rows of the score tile.
// All four waves compute the (cheap) scores of a 32-key tile; wave w owns value
// channels [128w, 128w+128), so a workgroup covers 512 of them and the key row
// is fetched from memory once: global -> registers (next tile prefetched) -> LDS
// row-major, then V^T is cut out of that LDS tile. Causal, optionally inside a
// sliding window or the token's block of positions; optional sink and sigmoid gate
// per head.
// Grid: (tokens x key splits, head chunks of 16 x value splits of 512, batch
// rows). With nks > 1 key splits a workgroup scans every nks-th run of tiles and
// leaves an unnormalised partial (fp32 values, running max, sum) in `ws`;
// latent_decode_merge_kernel folds the splits and the sink.
#define LD_KT 32
#define LD_VW 128                            // value channels per wave

template <int DKP>
__global__ void __launch_bounds__(256)
latent_decode_mfma_kernel(const bf16* __restrict__ q, long qstride, const bf16* __restrict__ kc,
                          long ktok, const int* __restrict__ pos, const int* __restrict__ seq,
                          const int* __restrict__ btab, int max_blocks,
                          const float* __restrict__ sink, bf16* __restrict__ out, int H, int Dk,
                          int Dv, int bsz, int S, float scale, int nsplit, int nks,
                          float* __restrict__ ws, int window, int cmask,
                          const bf16* __restrict__ gate, long gstride) {
    constexpr int KS = DKP + 8;
    constexpr int VS = LD_KT + 8;
    constexpr int VCH = 4 * LD_VW;
    extern __shared__ __attribute__((aligned(16))) uint16_t ld_lds[];
    uint16_t* k_lds = ld_lds;                            // LD_KT * KS
    uint16_t* vt_lds = ld_lds + LD_KT * KS;              // VCH * VS
    const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
    const int lr = lane & 15, lg = lane >> 4;
    const int b = blockIdx.z, t = blockIdx.x / nks, ksp = blockIdx.x % nks;
    const int h0 = (blockIdx.y / nsplit) * 16;
    const int dv0 = (blockIdx.y % nsplit) * VCH;         // this workgroup's first value channel
    const int dvn = min(VCH, Dv - dv0);
    if (seq[b] < 0) return;
    const int p = pos[(long)b * S + t];
    if (p < 0) return;                                   // uniform
    const int h = h0 + lr;                               // this lane's query row
    const bool hv = h < H;
    bf16x8_t qf[DKP / 32];
    {
        const bf16* qp = q + ((long)b * S + t) * qstride + (long)h * Dk;
#pragma unroll
        for (int ks = 0; ks < DKP / 32; ++ks) {
            uint4 raw = make_uint4(0, 0, 0, 0);
            if (hv && ks * 32 + lg * 8 < Dk) raw = *reinterpret_cast<const uint4*>(qp + ks * 32 + lg * 8);
            qf[ks] = *reinterpret_cast<bf16x8_t*>(&raw);
        }
    }
    const int* bt = btab + (long)b * max_blocks;
    // the token sees keys [first, p]; this split's keys [k_lo, n) are a
    // contiguous run of 32-key tiles counted from `first`
    const int first = max(max(0, p - window + 1), cmask > 0 ? (p / cmask) * cmask : 0);
    const int tiles = (p + 1 - first + LD_KT - 1) / LD_KT, per = (tiles + nks - 1) / nks;
    const int k_lo = first + ksp * per * LD_KT;
    const int n = min(p + 1, first + (ksp + 1) * per * LD_KT);
    float m_run = -INFINITY, l_run = 0.f;
    f32x4_t o_acc[LD_VW / 16];
#pragma unroll
    for (int nb = 0; nb < LD_VW / 16; ++nb) o_acc[nb] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    constexpr int NKI = (LD_KT * (DKP / 8) + 255) / 256;
    uint4 rk[NKI];
#define LD_FETCH(BASE)                                                                     \
    _Pragma("unroll") for (int x = 0; x < NKI; ++x) {                                      \
        const int c = tid + x * 256;                                                       \
        const int m = c / (DKP / 8), part = c % (DKP / 8);                                 \
        uint4 raw = make_uint4(0, 0, 0, 0);                                                \
        if (c < LD_KT * (DKP / 8) && (BASE) + m < n && part * 8 < Dk) {                    \
            const int j = (BASE) + m;                                                      \
            const int blk = bt[j / bsz];                                                   \
            const long slot = (long)(blk < 0 ? 0 : blk) * bsz + (j % bsz);                 \
            raw = *reinterpret_cast<const uint4*>(kc + slot * ktok + part * 8);            \
        }                                                                                  \
        rk[x] = raw;                                                                       \
    }
    LD_FETCH(k_lo)
    for (int base = k_lo; base < n; base += LD_KT) {
#pragma unroll
        for (int x = 0; x < NKI; ++x) {
            const int c = tid + x * 256;
            if (c < LD_KT * (DKP / 8))
                *reinterpret_cast<uint4*>(k_lds + (c / (DKP / 8)) * KS + (c % (DKP / 8)) * 8) = rk[x];
        }
        __syncthreads();
        if (base + LD_KT < n) LD_FETCH(base + LD_KT)     // in flight during the work below
        // ---- V^T (channels dv0..dv0+dvn) out of the K tile
        for (int c = tid; c < LD_KT * (VCH / 8); c += 256) {
            const int m = c % LD_KT, part = c / LD_KT;
            uint4 raw = make_uint4(0, 0, 0, 0);
            if (part * 8 < dvn) raw = *reinterpret_cast<const uint4*>(k_lds + m * KS + dv0 + part * 8);
            const uint32_t u[4] = {raw.x, raw.y, raw.z, raw.w};
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                vt_lds[(part * 8 + 2 * e) * VS + m] = (uint16_t)(u[e] & 0xffffu);
                vt_lds[(part * 8 + 2 * e + 1) * VS + m] = (uint16_t)(u[e] >> 16);
            }
        }
        // ---- S^T = K Q^T: lane gets keys 16*kb + 4*lg + r of row lr
        float sv[2][4];
        float mt = -INFINITY;
#pragma unroll
        for (int kb = 0; kb < 2; ++kb) {
            f32x4_t acc = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int ks = 0; ks < DKP / 32; ++ks) {
                const bf16x8_t ka = *reinterpret_cast<const bf16x8_t*>(
                    k_lds + (kb * 16 + lr) * KS + ks * 32 + lg * 8);
                acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ka, qf[ks], acc, 0, 0, 0);
            }
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int j = base + kb * 16 + lg * 4 + r;
                const float x = (j < n && hv) ? acc[r] * scale : -INFINITY;
                sv[kb][r] = x;
                mt = fmaxf(mt, x);
            }
        }
        mt = fmaxf(mt, __shfl_xor(mt, 16, WAVE));
        mt = fmaxf(mt, __shfl_xor(mt, 32, WAVE));
        const float m_new = fmaxf(m_run, mt);
        float corr = 1.f, psum = 0.f;
#pragma unroll
        for (int kb = 0; kb < 2; ++kb)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const float pv = (m_new > -INFINITY && sv[kb][r] > -INFINITY)
                    ? __expf(sv[kb][r] - m_new) : 0.f;
                sv[kb][r] = pv;
                psum += pv;
            }
        if (m_new > -INFINITY) corr = __expf(m_run - m_new);
        psum += __shfl_xor(psum, 16, WAVE);
        psum += __shfl_xor(psum, 32, WAVE);
        l_run = l_run * corr + psum;
        m_run = m_new;
        float cr[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) cr[r] = __shfl(corr, lg * 4 + r, WAVE);
#pragma unroll
        for (int nb = 0; nb < LD_VW / 16; ++nb)
#pragma unroll
            for (int r = 0; r < 4; ++r) o_acc[nb][r] *= cr[r];
        __syncthreads();                                 // V^T complete
        // ---- O += P V for this wave's 128 channels, P as hi + lo
        {
            struct { bf16x8_t v; } ph, pl;
#pragma unroll
            for (int jj = 0; jj < 8; ++jj) {
                const float pv = sv[jj >> 2][jj & 3];
                const __bf16 hb = (__bf16)pv;
                ph.v[jj] = hb;
                pl.v[jj] = (__bf16)(pv - (float)hb);
            }
#pragma unroll
            for (int nb = 0; nb < LD_VW / 16; ++nb) {
                union { bf16x8_t v; uint2 h2[2]; } vb;
                const uint16_t* vp = vt_lds + (wv * LD_VW + nb * 16 + lr) * VS + 4 * lg;
                vb.h2[0] = *reinterpret_cast<const uint2*>(vp);
                vb.h2[1] = *reinterpret_cast<const uint2*>(vp + 16);
                o_acc[nb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ph.v, vb.v, o_acc[nb], 0, 0, 0);
                o_acc[nb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pl.v, vb.v, o_acc[nb], 0, 0, 0);
            }
        }
        __syncthreads();
    }
#undef LD_FETCH
    if (nks > 1) {
        // partial result: [(token, head, split)][Dv values | max | sum]
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int hh = h0 + lg * 4 + r;
            const float mr = __shfl(m_run, lg * 4 + r, WAVE), lrn = __shfl(l_run, lg * 4 + r, WAVE);
            if (hh >= H) continue;
            float* wp = ws + ((((long)b * S + t) * H + hh) * nks + ksp) * (long)(Dv + 2);
#pragma unroll
            for (int nb = 0; nb < LD_VW / 16; ++nb) {
                const int d = wv * LD_VW + nb * 16 + lr;
                if (d < dvn) wp[dv0 + d] = o_acc[nb][r];
            }
            if (dv0 == 0 && wv == 0 && lr == 0) { wp[Dv] = mr; wp[Dv + 1] = lrn; }
        }
        return;
    }
    float fin = l_run > 0.f ? 1.f / l_run : 0.f;
    if (sink && hv) {
        const float sk = sink[h];
        const float mf = fmaxf(m_run, sk);
        const float ca = m_run > -INFINITY ? __expf(m_run - mf) : 0.f;
        fin = ca / (l_run * ca + __expf(sk - mf));
    }
    // one gate number per head
    if (gate && hv) fin *= sigmoidf_(__bfloat162float(gate[((long)b * S + t) * gstride + h]));
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        const int hh = h0 + lg * 4 + r;
        const float inv = __shfl(fin, lg * 4 + r, WAVE);
        if (hh >= H) continue;
        bf16* op = out + (((long)b * S + t) * H + hh) * (long)Dv + dv0 + wv * LD_VW;
#pragma unroll
        for (int nb = 0; nb < LD_VW / 16; ++nb) {
            const int d = wv * LD_VW + nb * 16 + lr;
            if (d < dvn) op[nb * 16 + lr] = __float2bfloat16(o_acc[nb][r] * inv);
        }
    }
}

// one wave per (token, head, LM_W value channels): out = sum_i o_i e^(m_i - M) / (sum_i l_i e^(m_i - M)
// + e^(sink - M)), M the largest of the splits' maxima and the sink
#define LM_W 128
__global__ void latent_decode_merge_kernel(const float* __restrict__ ws,
                                           const float* __restrict__ sink,
                                           const int* __restrict__ pos, const int* __restrict__ seq,
                                           bf16* __restrict__ out, long ntok, int S, int H, int Dv,
                                           int nks, const bf16* __restrict__ gate, long gstride) {
    const int lane = threadIdx.x & (WAVE - 1);
    const int parts = (Dv + LM_W - 1) / LM_W;
    const long id = (long)blockIdx.x * (blockDim.x / WAVE) + threadIdx.x / WAVE;
    const long wid = id / parts;
    const int d0 = (id % parts) * LM_W;
    if (wid >= ntok * H) return;
    const long tok = wid / H;
    const int h = wid % H;
    if (pos[tok] < 0 || seq[tok / S] < 0) return;
    const float* wp = ws + wid * nks * (long)(Dv + 2);
    const float sk = sink ? sink[h] : -INFINITY;
    float M = sk;
    for (int i = 0; i < nks; ++i) M = fmaxf(M, wp[i * (long)(Dv + 2) + Dv]);
    float L = sink ? expf(sk - M) : 0.f;
    for (int i = 0; i < nks; ++i) {
        const float mi = wp[i * (long)(Dv + 2) + Dv];
        if (mi > -INFINITY) L += wp[i * (long)(Dv + 2) + Dv + 1] * expf(mi - M);
    }
    float inv = L > 0.f ? 1.f / L : 0.f;
    if (gate) inv *= sigmoidf_(__bfloat162float(gate[tok * gstride + h]));
    float wgt[8];                                        // nks <= 8
#pragma unroll
    for (int i = 0; i < 8; ++i) {
        const float mi = i < nks ? wp[i * (long)(Dv + 2) + Dv] : -INFINITY;
        wgt[i] = mi > -INFINITY ? expf(mi - M) * inv : 0.f;
    }
#pragma unroll
    for (int d = d0 + lane; d < d0 + LM_W; d += WAVE) {
        if (d >= Dv) break;
        float o = 0.f;
#pragma unroll
        for (int i = 0; i < 8; ++i)
            if (i < nks) o += wp[i * (long)(Dv + 2) + d] * wgt[i];
        out[wid * Dv + d] = __float2bfloat16(o);
    }
}

// ------------------------------------------------------- gated delta rule
// Three kernels per step.
// (1) delta_prep_kernel, fully parallel over tokens: unit q and k per KV head
//     (q also scaled by D^-1/2), decay exp(-exp(A_log) softplus(a + dt_bias))
//     per head and key channel, beta = sigmoid(.), all fp32, into one row per
//     token: [q (G*D) | k (G*D) | decay (H*D) | beta (H)], stride PS.
// (2) gated_delta_kernel, the serial scan. Workgroup = (row, head, block of
//     value channels), 256 threads. The (D x Dv) state is kept in registers:
//     16 (8 for D <= 32) adjacent lanes share one value channel (column) and
//     split its D rows in float4-interleaved order, so a token costs D/16
//     multiply-adds per lane plus two DPP lane reductions and no
//     workgroup-wide traffic. Tokens go in chunks of TC through LDS; the next
//     chunk's rows are fetched into registers while the current one is
//     scanned. State memory layout is (slot, head, Dv, D): a lane's rows are
//     contiguous float4s, a column's rows one contiguous line.
// (3) gated_rmsnorm_kernel: per-head RMS norm, weight and sigmoid gate (needs
//     all value channels of a head, which (2) spreads over workgroups).
#define GD_THREADS 256

template <typename T>
__global__ void delta_prep_kernel(const float* __restrict__ qkv, long cstride,
                                  const T* __restrict__ beta, long bstride,
                                  const T* __restrict__ a, long astride,
                                  const float* __restrict__ dt_bias,
                                  const float* __restrict__ a_log, const int* __restrict__ pos,
                                  const int* __restrict__ seq, float* __restrict__ prep, long PS,
                                  long ntok, int S, int H, int G, int D, int per_head) {
    const int lane = threadIdx.x & (WAVE - 1);
    const int units = 2 * G + H;
    const long wid = (long)blockIdx.x * (blockDim.x / WAVE) + threadIdx.x / WAVE;
    if (wid >= ntok * units) return;
    const long tok = wid / units;
    const int u = wid % units;
    if (pos[tok] < 0 || seq[tok / S] < 0) return;
    float* pr = prep + tok * PS;
    if (u < 2 * G) {
        const float* src = qkv + tok * cstride + (long)u * D;      // q heads then k heads
        float ss = 0.f;
        for (int i = lane; i < D; i += WAVE) { float x = src[i]; ss += x * x; }
        float inv = 1.f / sqrtf(wave_sum(ss) + 1e-6f);
        if (u < G) inv *= 1.f / sqrtf((float)D);
        for (int i = lane; i < D; i += WAVE) pr[(long)u * D + i] = src[i] * inv;
        if (u < G) {
            // q^ . k^ of this KV head: lets the scan read out before it writes
            const float* ksrc = src + (long)G * D;
            float sk = 0.f, qk = 0.f;
            for (int i = lane; i < D; i += WAVE) { float y = ksrc[i]; sk += y * y; qk += src[i] * y; }
            sk = wave_sum(sk);
            qk = wave_sum(qk);
            if (lane == 0)
                pr[(long)(2 * G + H) * D + H + u] = qk * inv * (1.f / sqrtf(sk + 1e-6f));
        }
    } else {
        const int h = u - 2 * G;
        const float neg_rate = -expf(a_log[h]);
        if (per_head) {
            // one decay for the whole head, broadcast over its key channels
            const float dec = expf(neg_rate * softplusf_(ldf<T>(a + tok * astride + h) + dt_bias[h]));
            for (int i = lane; i < D; i += WAVE) pr[(long)(2 * G + h) * D + i] = dec;
        } else {
            const T* ap = a + tok * astride + (long)h * D;
            for (int i = lane; i < D; i += WAVE)
                pr[(long)(2 * G + h) * D + i] =
                    expf(neg_rate * softplusf_(ldf<T>(ap + i) + dt_bias[h * D + i]));
        }
        if (lane == 0)
            pr[(long)(2 * G + H) * D + h] = sigmoidf_(ldf<T>(beta + tok * bstride + h));
    }
}

// sum over the 8 or 16 adjacent lanes that share a value channel, on the DPP
// path (quad xor 1, quad xor 2, mirrored half row, mirrored row: after each
// step every lane of a group holds the group's sum, so any lane of the
// sibling group will do)
template <int PARTS>
DEV float part_sum(float v) {
    v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(
        0, __builtin_bit_cast(int, v), 0xB1, 0xF, 0xF, true));    // quad_perm [1,0,3,2]
    v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(
        0, __builtin_bit_cast(int, v), 0x4E, 0xF, 0xF, true));    // quad_perm [2,3,0,1]
    v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(
        0, __builtin_bit_cast(int, v), 0x141, 0xF, 0xF, true));   // row_half_mirror
    if (PARTS == 16)
        v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(
            0, __builtin_bit_cast(int, v), 0x140, 0xF, 0xF, true));   // row_mirror
    return v;
}

template <int DK, int TC, int GD_PARTS>
__global__ void __launch_bounds__(GD_THREADS)
gated_delta_kernel(const float* __restrict__ qkv, long cstride, const float* __restrict__ prep,
                   long PS, float* __restrict__ state, const int* __restrict__ pos,
                   const int* __restrict__ seq, const int* __restrict__ nvalid,
                   float* __restrict__ obuf, int S, int H, int G, int D, int Dv) {
    constexpr int GD_CW = GD_THREADS / GD_PARTS;   // value channels per workgroup
    constexpr int R = DK / GD_PARTS;         // rows per lane
    constexpr int F = R / 4;                 // float4s per lane
    constexpr int NQKG = 3 * TC * DK;        // LDS floats per chunk: q | k | decay
    constexpr int NE = NQKG + TC * GD_CW + 2 * TC;   // ... | v (TC x GD_CW) | beta | q.k
    constexpr int PER = (NE + GD_THREADS - 1) / GD_THREADS;
    __shared__ __attribute__((aligned(16))) float buf[PER * GD_THREADS];
    const float* qs = buf;
    const float* ks = buf + TC * DK;
    const float* gs = buf + 2 * TC * DK;
    const float* vs = buf + NQKG;
    const float* bs = vs + TC * GD_CW;
    const float* kqs = bs + TC;
    const int h = blockIdx.y, b = blockIdx.z;
    const int slot = seq[b];
    const int n = nvalid[b];
    if (slot < 0 || n <= 0) return;          // uniform over the workgroup
    const int tid = threadIdx.x;
    const int part = tid % GD_PARTS;
    const int cl = tid / GD_PARTS;
    const int col0 = blockIdx.x * GD_CW;
    const int col = col0 + cl;
    const bool act = col < Dv;
    const int g = h / (H / G);
    const int p0 = pos[(long)b * S];
    float* st = state + (((long)slot * H + h) * Dv + (act ? col : 0)) * D;
    float s[R];
#pragma unroll
    for (int f = 0; f < F; ++f)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int row = (f * GD_PARTS + part) * 4 + e;
            s[f * 4 + e] = (act && row < D && p0 > 0) ? st[row] : 0.f;
        }
    const long off_q = (long)g * D, off_k = (long)(G + g) * D, off_g = (long)(2 * G + h) * D;
    const long off_b = (long)(2 * G + H) * D + h;
    const long off_kq = (long)(2 * G + H) * D + H + g;
    const long off_v = 2L * G * D + (long)h * Dv + col0;

    float pre[PER];
    // chunk at t0 -> registers (loads are issued, not waited for)
#define GD_FETCH(T0)                                                                      \
    {                                                                                     \
        const int ftc = min(TC, n - (T0));                                                \
        const long frow = (long)b * S + (T0);                                             \
        _Pragma("unroll") for (int x = 0; x < PER; ++x) {                                 \
            const int idx = tid + x * GD_THREADS;                                         \
            float v = 0.f;                                                                \
            if (idx < NQKG) {                                                             \
                const int which = idx / (TC * DK), rem = idx % (TC * DK);                 \
                const int tk = rem / DK, i = rem % DK;                                    \
                if (tk < ftc && i < D)                                                    \
                    v = prep[(frow + tk) * PS + (which == 0 ? off_q : which == 1 ? off_k : off_g) + i]; \
            } else if (idx < NQKG + TC * GD_CW) {                                         \
                const int tk = (idx - NQKG) / GD_CW, c = (idx - NQKG) % GD_CW;            \
                if (tk < ftc && col0 + c < Dv) v = qkv[(frow + tk) * cstride + off_v + c]; \
            } else if (idx < NE) {                                                        \
                const int e = idx - NQKG - TC * GD_CW;                                    \
                const int tk = e % TC;                                                    \
                if (tk < ftc) v = prep[(frow + tk) * PS + (e < TC ? off_b : off_kq)];     \
            }                                                                             \
            pre[x] = v;                                                                   \
        }                                                                                 \
    }
    GD_FETCH(0)
    for (int t0 = 0; t0 < n; t0 += TC) {
        const int tc = min(TC, n - t0);
        const long row0 = (long)b * S + t0;
#pragma unroll
        for (int x = 0; x < PER; ++x) buf[tid + x * GD_THREADS] = pre[x];
        __syncthreads();
        if (t0 + TC < n) GD_FETCH(t0 + TC)   // in flight during the scan below
#pragma unroll 2
        for (int tk = 0; tk < tc; ++tk) {
            const float4* g4 = reinterpret_cast<const float4*>(gs + tk * DK) + part;
            const float4* k4 = reinterpret_cast<const float4*>(ks + tk * DK) + part;
            const float4* q4 = reinterpret_cast<const float4*>(qs + tk * DK) + part;
            float4 kk[F];
            float dot = 0.f, oq = 0.f;       // (dS)^T k and (dS)^T q, this lane's rows
#pragma unroll
            for (int f = 0; f < F; ++f) {
                const float4 gg = g4[f * GD_PARTS];
                const float4 qq = q4[f * GD_PARTS];
                kk[f] = k4[f * GD_PARTS];
                s[4 * f] *= gg.x; dot += s[4 * f] * kk[f].x; oq += s[4 * f] * qq.x;
                s[4 * f + 1] *= gg.y; dot += s[4 * f + 1] * kk[f].y; oq += s[4 * f + 1] * qq.y;
                s[4 * f + 2] *= gg.z; dot += s[4 * f + 2] * kk[f].z; oq += s[4 * f + 2] * qq.z;
                s[4 * f + 3] *= gg.w; dot += s[4 * f + 3] * kk[f].w; oq += s[4 * f + 3] * qq.w;
            }
            dot = part_sum<GD_PARTS>(dot);
            oq = part_sum<GD_PARTS>(oq);
            const float u = bs[tk] * (vs[tk * GD_CW + cl] - dot);
            // read-out of the updated state: (dS + k u^T)^T q = (dS)^T q + u (k.q)
            if (act && part == 0)
                obuf[((row0 + tk) * H + h) * (long)Dv + col] = oq + u * kqs[tk];
#pragma unroll
            for (int f = 0; f < F; ++f) {
                s[4 * f] += kk[f].x * u;
                s[4 * f + 1] += kk[f].y * u;
                s[4 * f + 2] += kk[f].z * u;
                s[4 * f + 3] += kk[f].w * u;
            }
        }
        __syncthreads();
    }
#undef GD_FETCH
    if (act) {
#pragma unroll
        for (int f = 0; f < F; ++f)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int row = (f * GD_PARTS + part) * 4 + e;
                if (row < D) st[row] = s[f * 4 + e];
            }
    }
}

// per-head RMS norm over the value channels, shared weight, sigmoid gate:
// one wave per (token, head); pad tokens produce zeros
template <typename T>
__global__ void gated_rmsnorm_kernel(const float* __restrict__ o, const T* __restrict__ gate,
                                     long gstride, const float* __restrict__ w, float eps,
                                     const int* __restrict__ pos, const int* __restrict__ seq,
                                     T* __restrict__ out, long ntok, int S, int H, int Dv,
                                     int gate_silu) {
    const int lane = threadIdx.x & (WAVE - 1);
    const long wid = (long)blockIdx.x * (blockDim.x / WAVE) + threadIdx.x / WAVE;
    if (wid >= ntok * H) return;
    const long tok = wid / H;
    const int h = wid % H;
    T* op = out + wid * Dv;
    if (pos[tok] < 0 || seq[tok / S] < 0) {
        for (int c = lane; c < Dv; c += WAVE) stf<T>(op + c, 0.f);
        return;
    }
    const float* ip = o + wid * Dv;
    float ss = 0.f;
    for (int c = lane; c < Dv; c += WAVE) { float v = ip[c]; ss += v * v; }
    const float inv = 1.f / sqrtf(wave_sum(ss) / Dv + eps);
    const T* gp = gate + tok * gstride + (long)h * Dv;
    for (int c = lane; c < Dv; c += WAVE) {
        const float gv = ldf<T>(gp + c);
        stf<T>(op + c, ip[c] * inv * w[c] * (gate_silu ? gv * sigmoidf_(gv) : sigmoidf_(gv)));
    }
}

// ------------------------------------------------------------- elementwise
template <typename T>
__global__ void softcap_kernel(const T* __restrict__ in, float* __restrict__ out, long n,
                               float cap) {
    for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < n;
         i += (long)gridDim.x * blockDim.x)
        out[i] = cap * tanhf(ldf<T>(in + i) / cap);
}

// x += sa*a (+ sb*b), fp32 residual stream
template <typename T>
__global__ void residual_add_kernel(float* __restrict__ x, const T* __restrict__ a, float sa,
                                    const T* __restrict__ b, float sb, long n) {
    for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < n;
         i += (long)gridDim.x * blockDim.x) {
        float v = x[i] + sa * ldf<T>(a + i);
        if (b) v += sb * ldf<T>(b + i);
        x[i] = v;
    }
}

// out[r, c] = gelu_tanh(gu[r, c]) * gu[r, I + c]
// gated units: act(gate) * up, act = the tanh form of gelu (0) or silu (1)
DEV float gelu_tanh_(float z) {
    return 0.5f * z * (1.f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}
template <int ACT> DEV float unit_act_(float z) { return ACT == 0 ? gelu_tanh_(z) : z * sigmoidf_(z); }

template <typename T, int ACT>
__global__ void gelu_mul_kernel(const T* __restrict__ gu, T* __restrict__ out, long rows, int I) {
    const long total = rows * I;
    for (long idx = (long)blockIdx.x * blockDim.x + threadIdx.x; idx < total;
         idx += (long)gridDim.x * blockDim.x) {
        const long r = idx / I;
        const int c = idx % I;
        const float z = ldf<T>(gu + r * 2 * I + c);
        const float u = ldf<T>(gu + r * 2 * I + I + c);
        stf<T>(out + idx, unit_act_<ACT>(z) * u);
    }
}

// 8 channels per thread, 16-byte accesses; rows on blockIdx.y (strided)
template <typename T, int ACT>
__global__ void gelu_mul_vec_kernel(const T* __restrict__ gu, T* __restrict__ out, long rows,
                                    int I) {
    const int c = (blockIdx.x * blockDim.x + threadIdx.x) * 8;
    if (c >= I) return;
    for (long r = blockIdx.y; r < rows; r += gridDim.y) {
        float z[8], u[8], o[8];
        load8<T>(gu + r * 2 * I + c, z);
        load8<T>(gu + r * 2 * I + I + c, u);
#pragma unroll
        for (int e = 0; e < 8; ++e) o[e] = unit_act_<ACT>(z[e]) * u[e];
        T* op = out + r * I + c;
        if constexpr (sizeof(T) == 2) {
            uint32_t pk[4];
#pragma unroll
            for (int e = 0; e < 4; ++e)
                pk[e] = (uint32_t)f2bf_rne(o[2 * e]) | ((uint32_t)f2bf_rne(o[2 * e + 1]) << 16);
            *reinterpret_cast<uint4*>(op) = make_uint4(pk[0], pk[1], pk[2], pk[3]);
        } else {
            *reinterpret_cast<float4*>(op) = make_float4(o[0], o[1], o[2], o[3]);
            *reinterpret_cast<float4*>(op + 4) = make_float4(o[4], o[5], o[6], o[7]);
        }
    }
}


// ------------------------------------------------------------------ RMS norm
// x / sqrt(mean(x^2) + eps) * w (or * (1 + w)); one 256-thread workgroup per
// row, fp32 statistics; input and output rows may be strided slices. The *_vec
// variants move 8 channels per thread with 16-byte accesses (widths that are
// multiples of 8 on 16-byte aligned rows); the second pass re-reads the row
// from cache, so any width works.
template <typename T> DEV void store8(T* p, const float* v);
template <> DEV void store8<float>(float* p, const float* v) {
    *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
    *reinterpret_cast<float4*>(p + 4) = make_float4(v[4], v[5], v[6], v[7]);
}
template <> DEV void store8<bf16>(bf16* p, const float* v) {
    uint32_t pk[4];
#pragma unroll
    for (int e = 0; e < 4; ++e)
        pk[e] = (uint32_t)f2bf_rne(v[2 * e]) | ((uint32_t)f2bf_rne(v[2 * e + 1]) << 16);
    *reinterpret_cast<uint4*>(p) = make_uint4(pk[0], pk[1], pk[2], pk[3]);
}

// 4 consecutive elements as floats, one 8- or 16-byte access
template <typename T> DEV void load4(const T* p, float* v);
template <> DEV void load4<bf16>(const bf16* p, float* v) {
    const uint2 raw = *reinterpret_cast<const uint2*>(p);
    v[0] = __uint_as_float(raw.x << 16); v[1] = __uint_as_float(raw.x & 0xffff0000u);
    v[2] = __uint_as_float(raw.y << 16); v[3] = __uint_as_float(raw.y & 0xffff0000u);
}
template <> DEV void load4<float>(const float* p, float* v) {
    const float4 a = *reinterpret_cast<const float4*>(p);
    v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w;
}
template <typename T> DEV void store4(T* p, const float* v);
template <> DEV void store4<float>(float* p, const float* v) {
    *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
}
template <> DEV void store4<bf16>(bf16* p, const float* v) {
    union { bf16 h[4]; uint2 u; } x;
#pragma unroll
    for (int e = 0; e < 4; ++e) x.h[e] = __float2bfloat16(v[e]);
    *reinterpret_cast<uint2*>(p) = x.u;
}

template <typename TIn, typename TOut>
__global__ void __launch_bounds__(LN_THREADS)
rms_norm_vec_kernel(const TIn* __restrict__ x, long xs, const float* __restrict__ w, int one_plus,
                    float eps, TOut* __restrict__ out, long os, int C) {
    __shared__ float red[LN_THREADS / WAVE];
    const long row = blockIdx.x;
    const TIn* xr = x + row * xs;
    float s = 0.f;
    for (int c = threadIdx.x * 8; c < C; c += LN_THREADS * 8) {
        float v[8];
        load8<TIn>(xr + c, v);
#pragma unroll
        for (int e = 0; e < 8; ++e) s += v[e] * v[e];
    }
    const float inv = 1.f / sqrtf(block_sum(s, red) / C + eps);
    TOut* o = out + row * os;
    const float add = one_plus ? 1.f : 0.f;
    for (int c = threadIdx.x * 8; c < C; c += LN_THREADS * 8) {
        float v[8], wv[8];
        load8<TIn>(xr + c, v);
        load8<float>(w + c, wv);
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] = v[e] * inv * (wv[e] + add);
        store8<TOut>(o + c, v);
    }
}

// post-norm residual step: stream[row] += rms_norm(v[row]) * (w | 1 + w) in fp32,
// v = y, or y + (sum of the row's `nc` coefficients) * extra (experts that pass
// their input through). `copy` (optional) receives the updated row in the next
// GEMM's input type, or, with `next_w`, the next sublayer's pre-norm
// rms_norm(updated row) * next_w: the row's new statistics come from the same
// pass that updates it.
template <typename TY, typename TC>
__global__ void __launch_bounds__(LN_THREADS)
add_rms_norm_vec_kernel(float* __restrict__ stream, const TY* __restrict__ y,
                        const float* __restrict__ w, int one_plus, float eps,
                        TC* __restrict__ copy, const TY* __restrict__ extra,
                        const float* __restrict__ coef, long cs, int nc,
                        const float* __restrict__ next_w, int C) {
    __shared__ float red[LN_THREADS / WAVE];
    const long row = blockIdx.x;
    const TY* yr = y + row * C;
    const TY* er = extra ? extra + row * C : nullptr;
    float cf = 0.f;
    if (er) for (int k = 0; k < nc; ++k) cf += coef[row * cs + k];
    float s = 0.f;
    for (int c = threadIdx.x * 8; c < C; c += LN_THREADS * 8) {
        float v[8];
        load8<TY>(yr + c, v);
        if (er) {
            float ev[8];
            load8<TY>(er + c, ev);
#pragma unroll
            for (int e = 0; e < 8; ++e) v[e] += cf * ev[e];
        }
#pragma unroll
        for (int e = 0; e < 8; ++e) s += v[e] * v[e];
    }
    const float inv = 1.f / sqrtf(block_sum(s, red) / C + eps);
    const float add = one_plus ? 1.f : 0.f;
    float* xr = stream + row * C;
    float s2 = 0.f;
    for (int c = threadIdx.x * 8; c < C; c += LN_THREADS * 8) {
        float v[8], wv[8], xv[8];
        load8<TY>(yr + c, v);
        if (er) {
            float ev[8];
            load8<TY>(er + c, ev);
#pragma unroll
            for (int e = 0; e < 8; ++e) v[e] += cf * ev[e];
        }
        load8<float>(w + c, wv);
        load8<float>(xr + c, xv);
#pragma unroll
        for (int e = 0; e < 8; ++e) { xv[e] += v[e] * inv * (wv[e] + add); s2 += xv[e] * xv[e]; }
        store8<float>(xr + c, xv);
        if (copy && !next_w) store8<TC>(copy + row * C + c, xv);
    }
    if (!copy || !next_w) return;                        // uniform
    __syncthreads();                                     // `red` is reused
    const float inv2 = 1.f / sqrtf(block_sum(s2, red) / C + eps);
    for (int c = threadIdx.x * 8; c < C; c += LN_THREADS * 8) {
        float xv[8], wv[8];
        load8<float>(xr + c, xv);                        // this thread's own stores
        load8<float>(next_w + c, wv);
#pragma unroll
        for (int e = 0; e < 8; ++e) xv[e] = xv[e] * inv2 * wv[e];
        store8<TC>(copy + row * C + c, xv);
    }
}

template <typename TIn, typename TOut>
__global__ void __launch_bounds__(LN_THREADS)
rms_norm_kernel(const TIn* __restrict__ x, long xs, const float* __restrict__ w, int one_plus,
                float eps, TOut* __restrict__ out, long os, int C) {
    __shared__ float red[LN_THREADS / WAVE];
    const long row = blockIdx.x;
    const TIn* xr = x + row * xs;
    float s = 0.f;
    for (int c = threadIdx.x; c < C; c += LN_THREADS) { const float v = ldf<TIn>(xr + c); s += v * v; }
    const float inv = 1.f / sqrtf(block_sum(s, red) / C + eps);
    TOut* o = out + row * os;
    const float add = one_plus ? 1.f : 0.f;
    for (int c = threadIdx.x; c < C; c += LN_THREADS)
        stf<TOut>(o + c, ldf<TIn>(xr + c) * inv * (w[c] + add));
}

// scalar form of add_rms_norm_vec_kernel (any width and alignment)
template <typename TY, typename TC>
__global__ void __launch_bounds__(LN_THREADS)
add_rms_norm_kernel(float* __restrict__ stream, const TY* __restrict__ y,
                    const float* __restrict__ w, int one_plus, float eps,
                    TC* __restrict__ copy, const TY* __restrict__ extra,
                    const float* __restrict__ coef, long cs, int nc,
                    const float* __restrict__ next_w, int C) {
    __shared__ float red[LN_THREADS / WAVE];
    const long row = blockIdx.x;
    const TY* yr = y + row * C;
    const TY* er = extra ? extra + row * C : nullptr;
    float cf = 0.f;
    if (er) for (int k = 0; k < nc; ++k) cf += coef[row * cs + k];
    float s = 0.f;
    for (int c = threadIdx.x; c < C; c += LN_THREADS) {
        const float v = ldf<TY>(yr + c) + (er ? cf * ldf<TY>(er + c) : 0.f);
        s += v * v;
    }
    const float inv = 1.f / sqrtf(block_sum(s, red) / C + eps);
    const float add = one_plus ? 1.f : 0.f;
    float* xr = stream + row * C;
    float s2 = 0.f;
    for (int c = threadIdx.x; c < C; c += LN_THREADS) {
        const float yv = ldf<TY>(yr + c) + (er ? cf * ldf<TY>(er + c) : 0.f);
        const float v = xr[c] + yv * inv * (w[c] + add);
        xr[c] = v;
        s2 += v * v;
        if (copy && !next_w) stf<TC>(copy + row * C + c, v);
    }
    if (!copy || !next_w) return;                        // uniform
    __syncthreads();
    const float inv2 = 1.f / sqrtf(block_sum(s2, red) / C + eps);
    for (int c = threadIdx.x; c < C; c += LN_THREADS)
        stf<TC>(copy + row * C + c, xr[c] * inv2 * next_w[c]);
}

// ----------------------------------------- residual step with the norm after the sum
// stream[row] = layer_norm(alpha * stream[row] + y[row]) * w + bias, fp32; `copy`
// (optional) receives the new row in the next GEMM's input type. One workgroup per
// row. The vector form keeps the row in registers between mean, variance (of the
// deviations) and output: one read of each operand, one write of each result.
template <typename TY, typename TC, int NV>
__global__ void __launch_bounds__(LN_THREADS)
add_layer_norm_vec_kernel(float* __restrict__ stream, const TY* __restrict__ y, float alpha,
                          const float* __restrict__ w, const float* __restrict__ bias, float eps,
                          TC* __restrict__ copy, int C) {
    __shared__ float red[LN_THREADS / WAVE];
    const long row = blockIdx.x;
    float* xr = stream + row * C;
    float v[NV][8];
    float s = 0.f;
#pragma unroll
    for (int j = 0; j < NV; ++j) {
        const int c = (j * LN_THREADS + threadIdx.x) * 8;
        if (c < C) {
            float yv[8];
            load8<float>(xr + c, v[j]);
            load8<TY>(y + row * C + c, yv);
#pragma unroll
            for (int e = 0; e < 8; ++e) { v[j][e] = alpha * v[j][e] + yv[e]; s += v[j][e]; }
        }
    }
    const float mean = block_sum(s, red) / C;
    float q = 0.f;
#pragma unroll
    for (int j = 0; j < NV; ++j)
        if ((j * LN_THREADS + threadIdx.x) * 8 < C)
#pragma unroll
            for (int e = 0; e < 8; ++e) { v[j][e] -= mean; q += v[j][e] * v[j][e]; }
    const float inv = 1.f / sqrtf(block_sum(q, red) / C + eps);
#pragma unroll
    for (int j = 0; j < NV; ++j) {
        const int c = (j * LN_THREADS + threadIdx.x) * 8;
        if (c >= C) continue;
        float wv[8], bv[8];
        load8<float>(w + c, wv);
        load8<float>(bias + c, bv);
#pragma unroll
        for (int e = 0; e < 8; ++e) v[j][e] = v[j][e] * inv * wv[e] + bv[e];
        store8<float>(xr + c, v[j]);
        if (copy) store8<TC>(copy + row * C + c, v[j]);
    }
}

// scalar form: any width and alignment (the sum is parked in the stream row)
template <typename TY, typename TC>
__global__ void __launch_bounds__(LN_THREADS)
add_layer_norm_kernel(float* __restrict__ stream, const TY* __restrict__ y, float alpha,
                      const float* __restrict__ w, const float* __restrict__ bias, float eps,
                      TC* __restrict__ copy, int C) {
    __shared__ float red[LN_THREADS / WAVE];
    const long row = blockIdx.x;
    float* xr = stream + row * C;
    float s = 0.f;
    for (int c = threadIdx.x; c < C; c += LN_THREADS) {
        const float v = alpha * xr[c] + ldf<TY>(y + row * C + c);
        xr[c] = v;                                       // re-read by this thread only
        s += v;
    }
    const float mean = block_sum(s, red) / C;
    float q = 0.f;
    for (int c = threadIdx.x; c < C; c += LN_THREADS) { const float d = xr[c] - mean; q += d * d; }
    const float inv = 1.f / sqrtf(block_sum(q, red) / C + eps);
    for (int c = threadIdx.x; c < C; c += LN_THREADS) {
        const float v = (xr[c] - mean) * inv * w[c] + bias[c];
        xr[c] = v;
        if (copy) stf<TC>(copy + row * C + c, v);
    }
}

// ---------------------------------------------------------- rotary positions
// pairs (2i, 2i+1) of the first 2*half channels of every head (split = 0), or
// pairs (i, i + half) (split = 1), turn by p * inv_freq[i] (fp32 angle, full-range
// sincosf); the rest is copied.
// One thread per (token, head, channel pair or trailing channel).
template <typename TIn, typename TOut>
__global__ void rope_pairs_kernel(const TIn* __restrict__ x, long xt, long xh,
                                  TOut* __restrict__ out, long ot, long oh,
                                  const int* __restrict__ pos, const float* __restrict__ inv_freq,
                                  int half, int split, long ntok, int N, int C) {
    const int per = half + (C - 2 * half);            // work items per head
    const long total = ntok * N * per;
    for (long idx = (long)blockIdx.x * blockDim.x + threadIdx.x; idx < total;
         idx += (long)gridDim.x * blockDim.x) {
        const int e = idx % per;
        const long th = idx / per;
        const int h = th % N;
        const long tok = th / N;
        const int p = pos[tok];
        const TIn* xp = x + tok * xt + (long)h * xh;
        TOut* op = out + tok * ot + (long)h * oh;
        if (e < half) {
            const int c0 = split ? e : 2 * e, c1 = split ? e + half : 2 * e + 1;
            float a = ldf<TIn>(xp + c0), b = ldf<TIn>(xp + c1);
            float sn, cs;
            sincosf((float)(p < 0 ? 0 : p) * inv_freq[e], &sn, &cs);
            stf<TOut>(op + c0, a * cs - b * sn);
            stf<TOut>(op + c1, b * cs + a * sn);
        } else {
            const int c = 2 * half + (e - half);
            stf<TOut>(op + c, ldf<TIn>(xp + c));
        }
    }
}

// ------------------------------------------------------- clamped gated unit
// out[r, c] = g * sigmoid(alpha * g) * (u + 1), g = min(gu[r, c], limit),
// u = clamp(gu[r, I + c], -limit, limit)
DEV float clamped_glu_(float g, float u, float limit, float alpha) {
    g = fminf(g, limit);
    u = fminf(fmaxf(u, -limit), limit);
    return g * sigmoidf_(alpha * g) * (u + 1.f);
}

template <typename T>
__global__ void clamped_glu_kernel(const T* __restrict__ gu, T* __restrict__ out, long rows, int I,
                                   float limit, float alpha) {
    const long total = rows * I;
    for (long idx = (long)blockIdx.x * blockDim.x + threadIdx.x; idx < total;
         idx += (long)gridDim.x * blockDim.x) {
        const long r = idx / I;
        const int c = idx % I;
        stf<T>(out + idx, clamped_glu_(ldf<T>(gu + r * 2 * I + c), ldf<T>(gu + r * 2 * I + I + c),
                                       limit, alpha));
    }
}

template <typename T>
__global__ void clamped_glu_vec_kernel(const T* __restrict__ gu, T* __restrict__ out, long rows,
                                       int I, float limit, float alpha) {
    const int c = (blockIdx.x * blockDim.x + threadIdx.x) * 8;
    if (c >= I) return;
    for (long r = blockIdx.y; r < rows; r += gridDim.y) {
        float z[8], u[8], o[8];
        load8<T>(gu + r * 2 * I + c, z);
        load8<T>(gu + r * 2 * I + I + c, u);
#pragma unroll
        for (int e = 0; e < 8; ++e) o[e] = clamped_glu_(z[e], u[e], limit, alpha);
        T* op = out + r * I + c;
        if constexpr (sizeof(T) == 2) {
            uint32_t pk[4];
#pragma unroll
            for (int e = 0; e < 4; ++e)
                pk[e] = (uint32_t)f2bf_rne(o[2 * e]) | ((uint32_t)f2bf_rne(o[2 * e + 1]) << 16);
            *reinterpret_cast<uint4*>(op) = make_uint4(pk[0], pk[1], pk[2], pk[3]);
        } else {
            *reinterpret_cast<float4*>(op) = make_float4(o[0], o[1], o[2], o[3]);
            *reinterpret_cast<float4*>(op + 4) = make_float4(o[4], o[5], o[6], o[7]);
        }
    }
}

// ------------------------------------------- per-head norm + half-split rotary
// One wave per (token, head): RMS norm over the head's C channels with a weight
// shared by the heads (optional), then rotary positions on the first 2*half
// channels, channel i paired with channel i + half, angle pos * inv_freq[i],
// cos and sin times mscale (half = 0: none). Statistics and angles are fp32;
// the normed row goes through LDS so a lane can read its partner channel.
#define HN_WAVES 4
#define HN_MAXC 512

template <typename TIn, typename TOut>
__global__ void __launch_bounds__(HN_WAVES * WAVE)
head_norm_rope_kernel(const TIn* __restrict__ x, long xt, long xh, TOut* __restrict__ out,
                      const int* __restrict__ pos, const float* __restrict__ nw, float eps,
                      const float* __restrict__ inv_freq, int half, float mscale,
                      long ntok, int N, int C) {
    __shared__ float rows[HN_WAVES][HN_MAXC];
    const int lane = threadIdx.x & (WAVE - 1), wv = threadIdx.x / WAVE;
    const long id = (long)blockIdx.x * HN_WAVES + wv;
    if (id >= ntok * N) return;
    const long tok = id / N;
    const int hd = id % N;
    const int p = pos[tok];
    TOut* op = out + (tok * N + hd) * (long)C;
    if (p < 0) {
        for (int c = lane; c < C; c += WAVE) stf<TOut>(op + c, 0.f);
        return;
    }
    const TIn* xp = x + tok * xt + (long)hd * xh;
    float* row = rows[wv];
    float ss = 0.f;
    for (int c = lane; c < C; c += WAVE) {
        const float v = ldf<TIn>(xp + c);
        row[c] = v;
        ss += v * v;
    }
    if (nw) {
        const float inv = 1.f / sqrtf(wave_sum(ss) / C + eps);
        for (int c = lane; c < C; c += WAVE) row[c] = row[c] * inv * nw[c];
    }
    __builtin_amdgcn_wave_barrier();
    // a lane owns whole pairs: one sincos serves both channels
    for (int i = lane; i < half; i += WAVE) {
        float sn, cs;
        sincosf((float)p * inv_freq[i], &sn, &cs);
        sn *= mscale; cs *= mscale;
        const float u = row[i], w2 = row[i + half];
        stf<TOut>(op + i, u * cs - w2 * sn);
        stf<TOut>(op + i + half, w2 * cs + u * sn);
    }
    for (int c = 2 * half + lane; c < C; c += WAVE) stf<TOut>(op + c, row[c]);
}

// ----------------------------------------------------- decayed linear recurrence
// S_t = a_t S_{t-1} + k_t (w_t v_t)^T, o_t = S_t^T q_t (+ skip_h v_t), one scalar
// decay per head and token, or (KIND 1) one per key channel: S_t = diag(a_t) S_{t-1} +
// k_t v_t^T. Workgroup = (row, head, 16 value channels); the 16
// lanes of a channel split its key rows (lane p owns rows p*R .. p*R+R-1), the
// state sits in registers for the whole step and is read/written once. Tokens
// are staged through LDS in chunks of DS_TC (q, k, v, decay, step size), so
// global loads are coalesced and the serial loop reads only LDS.
// Decay: selective (dt projection + dt_bias, a_log: w = softplus(dt + bias),
// a = exp(-exp(a_log) w)) or fixed per head (head_decay: a = decay, w = 1). KIND 1 takes
// `dt` (H*D wide, fp32) as the decays' logarithms. KIND 2: both are given per head and
// token, a = exp(dt), w = wgt, and the last of the Dv value channels is not read but one
// (a normalizer row).
//
// Long rows with few workgroups are cut into `nseg` segments of `seglen`
// tokens that run side by side; the recurrence is linear in the state, so
//   MODE 1: every segment scans from a ZERO state and leaves its end state E_c
//           and the product P_c of its decays (a scalar, or one per key channel) in
//           the workspace (no outputs);
//   decay_scan_link_kernel: start state of segment c, serially over the few
//           segments: S_c = P_{c-1} S_{c-1} + E_{c-1} (S_0 = the carried state);
//   MODE 2: every segment scans again from its true start state and writes
//           the outputs; the last one stores the carried state.
// MODE 0 is the plain single pass (decode steps, short portions, full batches).
#define DS_TC 16

template <typename T, typename TD, int R, int MODE, int KIND>
__global__ void __launch_bounds__(256)
decay_scan_kernel(const T* __restrict__ q, long qs, const T* __restrict__ k, long ks,
                  const T* __restrict__ v, long vs, const TD* __restrict__ dt, long dts,
                  const float* __restrict__ dt_bias, const float* __restrict__ a_log,
                  const float* __restrict__ head_decay, float k_scale,
                  const float* __restrict__ skip, float* __restrict__ state,
                  const int* __restrict__ pos, const int* __restrict__ seq,
                  const int* __restrict__ nvalid, float* __restrict__ out, int S, int H, int G,
                  int D, int Dv, float* __restrict__ ws, float* __restrict__ wdec, int nseg,
                  int seglen, const float* __restrict__ wgt) {
    constexpr int DP = 16 * R;
    constexpr bool CH = KIND == 1;
    __shared__ __attribute__((aligned(16))) float sd[CH ? DS_TC : 1][CH ? DP : 4];
    __shared__ __attribute__((aligned(16))) float sq[MODE == 1 ? 1 : DS_TC][DP], sk[DS_TC][DP];
    __shared__ float sv[DS_TC][16], sa[DS_TC], sw[DS_TC];
    const int b = blockIdx.z, h = blockIdx.y;
    const int sgi = MODE == 0 ? 0 : blockIdx.x % nseg;
    const int c0 = (MODE == 0 ? blockIdx.x : blockIdx.x / nseg) * 16;
    const int slot = seq[b];
    const int n = slot < 0 ? 0 : nvalid[b];
    if (n <= 0) return;                                   // uniform
    const int tid = threadIdx.x, part = tid & 15, cl = tid >> 4;
    const int c = c0 + cl;
    const bool cok = c < Dv;
    const int g = h / (H / G);
    const int p0 = pos[(long)b * S];
    const int tbeg = MODE == 0 ? 0 : min(n, sgi * seglen);
    const int tend = MODE == 0 ? n : min(n, tbeg + seglen);
    float* sp = state + (((long)slot * H + h) * Dv + (cok ? c : 0)) * (long)D;
    float* wp = MODE == 0 ? nullptr
        : ws + ((((long)b * nseg + sgi) * H + h) * Dv + (cok ? c : 0)) * (long)D;
    float st[R];
    const float* src = MODE == 0 ? (p0 > 0 ? sp : nullptr) : (MODE == 2 ? wp : nullptr);
    // a lane's rows are contiguous in memory too: 16-byte accesses when the
    // row length allows (every state row then starts on a 16-byte boundary)
    const bool v4 = (R % 4 == 0) && (D % 4 == 0);
    if (v4) {
#pragma unroll
        for (int r = 0; r < R; r += 4) {
            const int d = part * R + r;
            float4 s4 = make_float4(0.f, 0.f, 0.f, 0.f);
            if (cok && src && d < D) s4 = *reinterpret_cast<const float4*>(src + d);
            st[r] = s4.x; st[r + 1 < R ? r + 1 : r] = s4.y;
            st[r + 2 < R ? r + 2 : r] = s4.z; st[r + 3 < R ? r + 3 : r] = s4.w;
        }
    } else {
#pragma unroll
        for (int r = 0; r < R; ++r) {
            const int d = part * R + r;
            st[r] = (cok && src && d < D) ? src[d] : 0.f;
        }
    }
    const float skp = skip ? skip[h] : 0.f;
    float aprod[CH ? R : 1];
#pragma unroll
    for (int r = 0; r < (CH ? R : 1); ++r) aprod[r] = 1.f;
    for (int t0 = tbeg; t0 < tend; t0 += DS_TC) {
        const int cnt = min(DS_TC, tend - t0);
        __syncthreads();                                  // the previous chunk is consumed
        for (int idx = tid; idx < DS_TC * DP; idx += 256) {
            const int tt = idx / DP, d = idx % DP;
            float qv = 0.f, kv = 0.f;
            if (tt < cnt && d < D) {
                const long tok = (long)b * S + t0 + tt;
                if (MODE != 1) qv = ldf<T>(q + tok * qs + (long)g * D + d);
                kv = ldf<T>(k + tok * ks + (long)g * D + d) * k_scale;
            }
            if (MODE != 1) sq[tt][d] = qv;
            sk[tt][d] = kv;
            if constexpr (CH) {
                sd[tt][d] = (tt < cnt && d < D)
                    ? expf(ldf<TD>(dt + ((long)b * S + t0 + tt) * dts + (long)h * D + d)) : 0.f;
            }
        }
        {
            const int tt = tid >> 4, cc = tid & 15;       // 256 = DS_TC * 16
            float vv = 0.f;
            if (tt < cnt && c0 + cc < Dv)
                vv = KIND == 2 && c0 + cc == Dv - 1 ? 1.f
                    : ldf<T>(v + ((long)b * S + t0 + tt) * vs + (long)h * (Dv - (KIND == 2)) + c0 + cc);
            sv[tt][cc] = vv;
        }
        if (!CH && tid < cnt) {
            float a, w = 1.f;
            if constexpr (KIND == 2) {
                const long tok = (long)b * S + t0 + tid;
                w = wgt[tok * H + h];
                a = expf(ldf<TD>(dt + tok * dts + h));
            } else if (dt) {
                w = softplusf_(ldf<TD>(dt + ((long)b * S + t0 + tid) * dts + h) + dt_bias[h]);
                a = expf(-expf(a_log[h]) * w);
            } else {
                a = head_decay[h];
            }
            sa[tid] = a;
            sw[tid] = w;
        }
        __syncthreads();
        for (int tt = 0; tt < cnt; ++tt) {
            const float xv = sv[tt][cl];
            const float wv = CH ? xv : sw[tt] * xv;
            float ar[R];                                  // this lane's decays
            if constexpr (!CH) {
                const float a = sa[tt];
#pragma unroll
                for (int r = 0; r < R; ++r) ar[r] = a;
            } else if constexpr (R % 4 == 0) {
#pragma unroll
                for (int r = 0; r < R; r += 4) {
                    const float4 a4 = *reinterpret_cast<const float4*>(&sd[tt][part * R + r]);
                    ar[r] = a4.x; ar[r + 1] = a4.y; ar[r + 2] = a4.z; ar[r + 3] = a4.w;
                }
            } else {
#pragma unroll
                for (int r = 0; r < R; ++r) ar[r] = sd[tt][part * R + r];
            }
            // a lane's key rows are contiguous: 16-byte LDS reads
            float kr[R], qr[R];
            if constexpr (R % 4 == 0) {
#pragma unroll
                for (int r = 0; r < R; r += 4) {
                    const float4 k4 = *reinterpret_cast<const float4*>(&sk[tt][part * R + r]);
                    kr[r] = k4.x; kr[r + 1] = k4.y; kr[r + 2] = k4.z; kr[r + 3] = k4.w;
                    if (MODE != 1) {
                        const float4 q4 = *reinterpret_cast<const float4*>(&sq[tt][part * R + r]);
                        qr[r] = q4.x; qr[r + 1] = q4.y; qr[r + 2] = q4.z; qr[r + 3] = q4.w;
                    }
                }
            } else {
#pragma unroll
                for (int r = 0; r < R; ++r) {
                    kr[r] = sk[tt][part * R + r];
                    if (MODE != 1) qr[r] = sq[tt][part * R + r];
                }
            }
            if (MODE == 1) {
#pragma unroll
                for (int r = 0; r < (CH ? R : 1); ++r) aprod[r] *= ar[r];
#pragma unroll
                for (int r = 0; r < R; ++r) st[r] = ar[r] * st[r] + kr[r] * wv;
            } else {
                float acc = 0.f;
#pragma unroll
                for (int r = 0; r < R; ++r) {
                    st[r] = ar[r] * st[r] + kr[r] * wv;
                    acc += st[r] * qr[r];
                }
                acc += __shfl_xor(acc, 8, WAVE);
                acc += __shfl_xor(acc, 4, WAVE);
                acc += __shfl_xor(acc, 2, WAVE);
                acc += __shfl_xor(acc, 1, WAVE);
                if (part == 0 && cok)
                    out[(((long)b * S + t0 + tt) * H + h) * (long)Dv + c] = acc + skp * xv;
            }
        }
    }
    if (MODE == 1 && c0 == 0) {
        const long wi = ((long)b * nseg + sgi) * H + h;
        if constexpr (CH) {
            if (cl == 0) {
#pragma unroll
                for (int r = 0; r < R; ++r)
                    if (part * R + r < D) wdec[wi * D + part * R + r] = aprod[r];
            }
        } else if (tid == 0) {
            wdec[wi] = aprod[0];
        }
    }
    float* dst = MODE == 1 ? wp : ((MODE == 0 || sgi == nseg - 1) ? sp : nullptr);
    if (cok && dst) {
        if (v4) {
#pragma unroll
            for (int r = 0; r < R; r += 4) {
                const int d = part * R + r;
                if (d < D)
                    *reinterpret_cast<float4*>(dst + d) = make_float4(
                        st[r], st[r + 1 < R ? r + 1 : r], st[r + 2 < R ? r + 2 : r],
                        st[r + 3 < R ? r + 3 : r]);
            }
        } else {
#pragma unroll
            for (int r = 0; r < R; ++r) {
                const int d = part * R + r;
                if (d < D) dst[d] = st[r];
            }
        }
    }
}

// start states of the segments, in place over their end states (see above)
__global__ void decay_scan_link_kernel(float* __restrict__ ws, const float* __restrict__ wdec,
                                       const float* __restrict__ state,
                                       const int* __restrict__ pos, const int* __restrict__ seq,
                                       const int* __restrict__ nvalid, int B, int S, int H,
                                       long per_head, int nseg, int dch) {
    // dch: decay channels (1: a scalar per head, else the key dimension)
    const long total = (long)B * H * per_head;
    for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < total;
         i += (long)gridDim.x * blockDim.x) {
        const long e = i % per_head;
        const int h = (i / per_head) % H;
        const int b = i / (per_head * H);
        const int slot = seq[b];
        if (slot < 0 || nvalid[b] <= 0) continue;
        float s = pos[(long)b * S] > 0 ? state[((long)slot * H + h) * per_head + e] : 0.f;
        for (int c = 0; c < nseg; ++c) {
            float* p = ws + (((long)b * nseg + c) * H + h) * per_head + e;
            const float end = *p;
            *p = s;
            s = wdec[(((long)b * nseg + c) * H + h) * dch + (dch > 1 ? e % dch : 0)] * s + end;
        }
    }
}

// ------------------------------------------------- low-rank channel decays
// log decay of a key channel: log(sigmoid(low[t] . w[c] + bias[c])) * inv_tau, all
// fp32 (a very negative logit does not underflow). A thread owns one channel for
// LRD_T tokens (few in steps of few tokens), whose low-rank rows sit in LDS.
#define LRD_R 64

template <typename T, int LRD_T>
__global__ void __launch_bounds__(256)
low_rank_decay_kernel(const T* __restrict__ low, long ls, const T* __restrict__ w, int vec,
                      const float* __restrict__ bias, float inv_tau, float* __restrict__ out,
                      long rows, int C, int rank) {
    __shared__ float sl[LRD_T][LRD_R];
    const int c = blockIdx.x * 256 + threadIdx.x;
    for (long t0 = (long)blockIdx.y * LRD_T; t0 < rows; t0 += (long)gridDim.y * LRD_T) {
        float acc[LRD_T];
        const float b0 = c < C ? bias[c] : 0.f;
#pragma unroll
        for (int t = 0; t < LRD_T; ++t) acc[t] = b0;
        for (int r0 = 0; r0 < rank; r0 += LRD_R) {
            const int rn = min(LRD_R, rank - r0);
            __syncthreads();
            for (int i = threadIdx.x; i < LRD_T * LRD_R; i += 256) {
                const int t = i / LRD_R, r = i % LRD_R;
                sl[t][r] = (t0 + t < rows && r < rn) ? ldf<T>(low + (t0 + t) * ls + r0 + r) : 0.f;
            }
            __syncthreads();
            if (c < C) {
                for (int r = 0; r < rn; r += 8) {
                    float wv[8];
                    const T* wp = w + (long)c * rank + r0 + r;
                    if (vec) {
                        load8<T>(wp, wv);
                    } else {
#pragma unroll
                        for (int e = 0; e < 8; ++e) wv[e] = r + e < rn ? ldf<T>(wp + e) : 0.f;
                    }
#pragma unroll
                    for (int t = 0; t < LRD_T; ++t)
#pragma unroll
                        for (int e = 0; e < 8; ++e) acc[t] += wv[e] * sl[t][r + e];
                }
            }
        }
        if (c < C) {
#pragma unroll
            for (int t = 0; t < LRD_T; ++t)
                if (t0 + t < rows) {
                    const float z = acc[t];
                    out[(t0 + t) * C + c] = (fminf(z, 0.f) - log1pf(expf(-fabsf(z)))) * inv_tau;
                }
        }
    }
}

// --------------------------- channel-decay recurrence in chunks, matrix cores
// The recurrence of decay_scan_kernel<CH> for rows of many tokens, bf16 inputs, cut
// into chunks of 64 tokens (4 sub-blocks of 16). With G the running sum of log
// decays, token s reaches token t >= s through exp(G_t - G_s) per key channel:
//   gla_chunk_state_kernel  E_c = sum_s k_s exp(G_end - G_s) v_s^T and exp(G_end)
//                           of every chunk on its own;
//   gla_chunk_link_kernel   serially over the chunks: start state of each (in place
//                           over E_c) and the carried state;
//   gla_chunk_out_kernel    o_t = (q_t exp(G_t)) S_c + sum_{s <= t} A_ts v_s, then the
//                           per-head RMS norm, its weight and the silu gate.
// Every exponent is taken relative to a sub-block's edge between the two tokens, so
// it is never positive: no overflow, whatever the decays. A_ts of two different
// sub-blocks is a product of two such factors (matrix cores), and so it is inside a
// sub-block whose decays are mild; otherwise it is summed directly in fp32. fp32 operands of the matrix cores are split into bf16
// terms: three for the keys that enter the state (24 bits), two elsewhere (16 bits);
// accumulation and state are fp32.
#define GC_N 64
#define GC_VS (GC_N + 8)

DEV float exp2_(float x) { return __builtin_amdgcn_exp2f(x); }   // hardware, 1 ulp

DEV void split_bf16_(float x, __bf16& hi, __bf16& lo) {
    hi = (__bf16)x;
    lo = (__bf16)(x - (float)hi);
}

// 64 token rows of P*8 bf16 channels each, 16 bytes a time, into registers: all loads
// are in flight together (addresses are clamped, not branched around), zeros past the
// last token (cnt >= 1) and channel (n, a multiple of 8)
template <int P>
DEV void gc_load_rows_(const bf16* __restrict__ x, long xs, int cnt, int n, uint4* r, int tid) {
#pragma unroll
    for (int i = 0; i < P / 4; ++i) {
        const int c = tid + i * 256, m = c % GC_N, part = c / GC_N;
        const uint4 v = *reinterpret_cast<const uint4*>(
            x + (long)min(m, cnt - 1) * xs + min(part * 8, n - 8));
        const bool ok = m < cnt && part * 8 < n;
        r[i] = make_uint4(ok ? v.x : 0, ok ? v.y : 0, ok ? v.z : 0, ok ? v.w : 0);
    }
}
// registers of gc_load_rows_ -> V^T (P*8 channels, GC_VS)
template <int P>
DEV void gc_store_vt_(const uint4* r, uint16_t* __restrict__ vt, int tid) {
#pragma unroll
    for (int i = 0; i < P / 4; ++i) {
        const int c = tid + i * 256, m = c % GC_N, part = c / GC_N;
        const uint32_t u[4] = {r[i].x, r[i].y, r[i].z, r[i].w};
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            vt[(part * 8 + 2 * e) * GC_VS + m] = (uint16_t)(u[e] & 0xffffu);
            vt[(part * 8 + 2 * e + 1) * GC_VS + m] = (uint16_t)(u[e] >> 16);
        }
    }
}

template <int DP, int NT>
__global__ void __launch_bounds__(256)
gla_chunk_state_kernel(const bf16* __restrict__ k, long ks, const bf16* __restrict__ v, long vs,
                       const float* __restrict__ ld, float k_scale, const int* __restrict__ pos,
                       const int* __restrict__ seq, const int* __restrict__ nvalid,
                       float* __restrict__ ws, float* __restrict__ wdec, int S, int H, int D,
                       int Dv, int nc) {
    __shared__ __attribute__((aligned(16))) uint16_t kt[3][DP * GC_VS];
    __shared__ __attribute__((aligned(16))) uint16_t vt[NT * 16 * GC_VS];
    __shared__ float tot[4][DP];
    const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
    const int lr = lane & 15, lg = lane >> 4;
    const int c = blockIdx.x % nc, d0 = blockIdx.x / nc * DP, h = blockIdx.y, b = blockIdx.z;
    const int n = seq[b] < 0 ? 0 : nvalid[b];
    const int cnt = min(GC_N, n - c * GC_N);
    if (cnt <= 0) return;                                 // uniform
    const long tok0 = (long)b * S + c * GC_N;
    const int Dn = min(DP, D - d0);                       // this workgroup's key channels
    const float* lp = ld + (long)h * D + d0;
    const bf16* kp = k + (long)h * D + d0;
    const long lst = (long)H * D;
    // one (channel, sub-block of 16 tokens) task per thread
    static_assert(4 * DP <= 256, "one task per thread");
    uint4 vr[NT / 2];
    gc_load_rows_<NT * 2>(v + tok0 * vs + (long)h * Dv, vs, cnt, Dv, vr, tid);
    const int d = tid % DP, sb = tid / DP;
    float g[16], kv[16];
    if (sb < 4) {
        float t = 0.f;
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            const int m = sb * 16 + i;
            const bool ok = m < cnt && d < Dn;
            const long tk = tok0 + min(m, cnt - 1);
            const int dc = min(d, Dn - 1);
            const float gv = lp[tk * lst + dc], kk = ldf<bf16>(kp + tk * ks + dc);
            g[i] = ok ? gv : 0.f;
            kv[i] = ok ? kk * k_scale : 0.f;
        }
#pragma unroll
        for (int i = 0; i < 16; ++i) t += g[i];
        tot[sb][d] = t;
    }
    gc_store_vt_<NT * 2>(vr, vt, tid);
    __syncthreads();
    if (sb < 4) {
        float after = 0.f;                                // decays of the later tokens
        for (int m = sb + 1; m < 4; ++m) after += tot[m][d];
        bf16x8_t t0[2], t1[2], t2[2];                     // the three terms of 16 tokens
#pragma unroll
        for (int i = 15; i >= 0; --i) {
            const float x = kv[i] * expf(after);
            after += g[i];
            const __bf16 a0 = (__bf16)x;
            const float r1 = x - (float)a0;
            const __bf16 a1 = (__bf16)r1;
            t0[i >> 3][i & 7] = a0;
            t1[i >> 3][i & 7] = a1;
            t2[i >> 3][i & 7] = (__bf16)(r1 - (float)a1);
        }
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            const int at = d * GC_VS + sb * 16 + u * 8;
            *reinterpret_cast<bf16x8_t*>(kt[0] + at) = t0[u];
            *reinterpret_cast<bf16x8_t*>(kt[1] + at) = t1[u];
            *reinterpret_cast<bf16x8_t*>(kt[2] + at) = t2[u];
        }
        if (sb == 0 && d < Dn) wdec[(((long)b * nc + c) * H + h) * D + d0 + d] = expf(after);
    }
    __syncthreads();
    float* wp = ws + (((long)b * nc + c) * H + h) * (long)Dv * D + d0;
    constexpr int DT = DP / 16;
    for (int tile = wv; tile < DT * NT; tile += 4) {
        const int dt = tile % DT, nt = tile / DT;
        if (nt * 16 >= Dv || dt * 16 >= Dn) continue;
        f32x4_t acc = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kk = 0; kk < 2; ++kk) {
            const bf16x8_t va = *reinterpret_cast<const bf16x8_t*>(
                vt + (nt * 16 + lr) * GC_VS + kk * 32 + lg * 8);
#pragma unroll
            for (int e = 2; e >= 0; --e) {                // small terms first
                const bf16x8_t kb = *reinterpret_cast<const bf16x8_t*>(
                    kt[e] + (dt * 16 + lr) * GC_VS + kk * 32 + lg * 8);
                acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(va, kb, acc, 0, 0, 0);
            }
        }
        const int dd = dt * 16 + lr;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int nn = nt * 16 + lg * 4 + r;
            if (nn < Dv && dd < Dn) wp[(long)nn * D + dd] = acc[r];
        }
    }
}

// start states of the chunks, in place over their contributions, and the carried
// state (dch: decay channels, the key dimension or 1); eight chunks' loads are in
// flight at a time. A start state leaves as its two
// bf16 terms (the high one in the high half of the word), ready for the read-out.
__global__ void __launch_bounds__(256)
gla_chunk_link_kernel(float* __restrict__ ws, const float* __restrict__ wdec,
                      float* __restrict__ state, const int* __restrict__ pos,
                      const int* __restrict__ seq, const int* __restrict__ nvalid, int B, int S,
                      int H, int dch, long per_head, int nc) {
    const long total = (long)B * H * per_head;
    for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < total;
         i += (long)gridDim.x * blockDim.x) {
        const long e = i % per_head;
        const int h = (i / per_head) % H, b = i / (per_head * H), d = dch > 1 ? e % dch : 0;
        const int slot = seq[b], n = slot < 0 ? 0 : nvalid[b];
        if (n <= 0) continue;
        const int chunks = (n + GC_N - 1) / GC_N;
        float* sp = state + ((long)slot * H + h) * per_head + e;
        float s = pos[(long)b * S] > 0 ? *sp : 0.f;
        float* wp = ws + ((long)b * nc * H + h) * per_head + e;
        const float* dp = wdec + ((long)b * nc * H + h) * dch + d;
        const long wst = (long)H * per_head, dst = (long)H * dch;
        for (int c0 = 0; c0 < chunks; c0 += 8) {
            float en[8], dc[8];
#pragma unroll
            for (int j = 0; j < 8; ++j)
                if (c0 + j < chunks) { en[j] = wp[(c0 + j) * wst]; dc[j] = dp[(c0 + j) * dst]; }
#pragma unroll
            for (int j = 0; j < 8; ++j)
                if (c0 + j < chunks) {
                    __bf16 hi, lo;
                    split_bf16_(s, hi, lo);
                    wp[(c0 + j) * wst] = __uint_as_float(
                        ((uint32_t)__builtin_bit_cast(uint16_t, hi) << 16) |
                        __builtin_bit_cast(uint16_t, lo));
                    s = dc[j] * s + en[j];
                }
        }
        *sp = s;
    }
}

template <int DP, int NT>
__global__ void __launch_bounds__(256, 2)
gla_chunk_out_kernel(const bf16* __restrict__ q, long qs, const bf16* __restrict__ k, long ks,
                     const bf16* __restrict__ v, long vs, const float* __restrict__ ld,
                     float k_scale, const bf16* __restrict__ gate, long gs,
                     const float* __restrict__ nw, float eps, const int* __restrict__ seq,
                     const int* __restrict__ nvalid, const float* __restrict__ ws,
                     bf16* __restrict__ out, int S, int H, int D, int Dv, int nc) {
    constexpr int KS = DP + 8, LS = DP + 4, KK = DP / 32;
    extern __shared__ __attribute__((aligned(16))) float smem[];
    float* ll = smem;                                     // GC_N * LS: running log decay in a sub-block
    float (*tot)[DP] = reinterpret_cast<float (*)[DP]>(ll + GC_N * LS);         // 4 x DP
    uint16_t* kl = reinterpret_cast<uint16_t*>(ll + GC_N * LS + 4 * DP);        // GC_N * KS
    uint16_t* vt = kl + GC_N * KS;                                              // NT * 16 * GC_VS
    const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6;    // wave = sub-block
    const int lr = lane & 15, lg = lane >> 4;
    const int c = blockIdx.x, h = blockIdx.y, b = blockIdx.z;
    const int n = seq[b] < 0 ? 0 : nvalid[b];
    const int cnt = min(GC_N, n - c * GC_N);
    if (cnt <= 0) return;                                 // uniform
    const long tok0 = (long)b * S + c * GC_N;
    const bool tv = w * 16 + lr < cnt;
    // this lane's query row (token 16 w + lr), channels kk*32 + lg*8 ..
    uint4 qr[KK];
#pragma unroll
    for (int kk = 0; kk < KK; ++kk) {
        const int d = kk * 32 + lg * 8;
        qr[kk] = make_uint4(0, 0, 0, 0);
        if (tv && d < D)
            qr[kk] = *reinterpret_cast<const uint4*>(q + (tok0 + w * 16 + lr) * qs + (long)h * D + d);
    }
    // start state, this lane's rows (value channel lr of every tile), packed terms:
    // the first block of key channels is fetched here, the next ones while one is used
    const float* sp = ws + (((long)b * nc + c) * H + h) * (long)Dv * D + (long)lr * D + lg * 8;
    uint4 sr[NT][2];
#define GC_FETCH(KKI)                                                                      \
    _Pragma("unroll") for (int nt = 0; nt < NT; ++nt) {                                    \
        sr[nt][0] = sr[nt][1] = make_uint4(0, 0, 0, 0);                                    \
        if (nt * 16 + lr < Dv && (KKI) * 32 + lg * 8 < D) {                                \
            const float* rp = sp + (long)nt * 16 * D + (KKI) * 32;                         \
            sr[nt][0] = *reinterpret_cast<const uint4*>(rp);                               \
            sr[nt][1] = *reinterpret_cast<const uint4*>(rp + 4);                           \
        }                                                                                  \
    }
    GC_FETCH(0)
    uint4 vr[NT / 2], kr[DP / 32];
    gc_load_rows_<NT * 2>(v + tok0 * vs + (long)h * Dv, vs, cnt, Dv, vr, tid);
    gc_load_rows_<DP / 8>(k + tok0 * ks + (long)h * D, ks, cnt, D, kr, tid);
    constexpr int TASKS = (4 * DP + 255) / 256;           // (channel, sub-block) per thread
    float g[TASKS][16];
#pragma unroll
    for (int x = 0; x < TASKS; ++x) {
        const int task = tid + x * 256, d = min(task % DP, D - 1), sb = task / DP;
#pragma unroll
        for (int i = 0; i < 16; ++i)
            g[x][i] = ld[(tok0 + min(sb * 16 + i, cnt - 1)) * (long)(H * D) + (long)h * D + d];
    }
    gc_store_vt_<NT * 2>(vr, vt, tid);
#pragma unroll
    for (int i = 0; i < DP / 32; ++i) {
        const int x = tid + i * 256;
        *reinterpret_cast<uint4*>(kl + (x % GC_N) * KS + (x / GC_N) * 8) = kr[i];
    }
#pragma unroll
    for (int x = 0; x < TASKS; ++x) {
        const int task = tid + x * 256, d = task % DP, sb = task / DP;
        if (sb >= 4) continue;                            // DP = 32: half the threads
        float t = 0.f;
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            // base 2 from here on; tokens past the last and padding channels stand still
            t += (sb * 16 + i < cnt && d < D) ? g[x][i] * 1.4426950408889634f : 0.f;
            ll[(sb * 16 + i) * LS + d] = t;
        }
        tot[sb][d] = t;
    }
    __syncthreads();
    if (w * 16 >= cnt) return;                            // no barriers below
    float qf[KK][8], lt[KK][8], pre[KK][8];               // q, L_t, log decays of earlier sub-blocks
#pragma unroll
    for (int kk = 0; kk < KK; ++kk) {
        const int d = kk * 32 + lg * 8;
        const uint32_t u[4] = {qr[kk].x, qr[kk].y, qr[kk].z, qr[kk].w};
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            qf[kk][e] = __uint_as_float(e & 1 ? u[e / 2] & 0xffff0000u : u[e / 2] << 16);
            lt[kk][e] = ll[(w * 16 + lr) * LS + d + e];
            float pr = 0.f;
            for (int m = 0; m < w; ++m) pr += tot[m][d + e];
            pre[kk][e] = pr;
        }
    }
    f32x4_t o[NT];
#pragma unroll
    for (int nt = 0; nt < NT; ++nt) o[nt] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    // ---- (q exp(G_t)) S: S rows (value channel lr of the tile) from memory
    {
#pragma unroll
        for (int kk = 0; kk < KK; ++kk) {
            bf16x8_t qh, ql;
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                __bf16 hi, lo;
                split_bf16_(qf[kk][e] * exp2_(pre[kk][e] + lt[kk][e]), hi, lo);
                qh[e] = hi; ql[e] = lo;
            }
#pragma unroll
            for (int nt = 0; nt < NT; ++nt) {
                const uint4 s0 = sr[nt][0], s1 = sr[nt][1];
                // two words (hi | lo) each -> a pair of high and a pair of low terms
                const uint4 hv = make_uint4(
                    (s0.x >> 16) | (s0.y & 0xffff0000u), (s0.z >> 16) | (s0.w & 0xffff0000u),
                    (s1.x >> 16) | (s1.y & 0xffff0000u), (s1.z >> 16) | (s1.w & 0xffff0000u));
                const uint4 lv = make_uint4(
                    (s0.x & 0xffffu) | (s0.y << 16), (s0.z & 0xffffu) | (s0.w << 16),
                    (s1.x & 0xffffu) | (s1.y << 16), (s1.z & 0xffffu) | (s1.w << 16));
                const bf16x8_t sh = __builtin_bit_cast(bf16x8_t, hv);
                const bf16x8_t sl = __builtin_bit_cast(bf16x8_t, lv);
                o[nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ql, sh, o[nt], 0, 0, 0);
                o[nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qh, sl, o[nt], 0, 0, 0);
                o[nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qh, sh, o[nt], 0, 0, 0);
            }
            if (kk + 1 < KK) GC_FETCH(kk + 1)
        }
    }
#undef GC_FETCH
    // ---- A^T: lane gets keys 4*lg + r of sub-block j for query lr
    float sc[4][4];
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int r = 0; r < 4; ++r) sc[j][r] = 0.f;
    // Own sub-block: when no channel decays by more than 2^-60 inside it, exp(L_t) and
    // exp(-L_s) are both far from overflow and the product form below serves it too
    // (what it gives for s > t is dropped); else exp(L_t - L_s) is taken directly,
    // channels split over the four lane groups.
    bool mild = true;
#pragma unroll
    for (int kk = 0; kk < KK; ++kk)
#pragma unroll
        for (int e = 0; e < 8; ++e) mild = mild && tot[w][kk * 32 + lg * 8 + e] > -60.f;
    mild = __all(mild);
    if (!mild) {
        float part[16];
#pragma unroll
        for (int si = 0; si < 16; ++si) {
            float a = 0.f;
#pragma unroll
            for (int kk = 0; kk < KK; ++kk) {
                const int d = kk * 32 + lg * 8;
                float kv[8], lv[8];
                load8<bf16>(reinterpret_cast<const bf16*>(kl) + (w * 16 + si) * KS + d, kv);
                load8<float>(ll + (w * 16 + si) * LS + d, lv);
#pragma unroll
                for (int e = 0; e < 8; ++e)
                    a += qf[kk][e] * kv[e] * exp2_(lt[kk][e] - lv[e]);   // s > t: dropped below
            }
            part[si] = a;
        }
#pragma unroll
        for (int si = 0; si < 16; ++si) {
            part[si] += __shfl_xor(part[si], 16, WAVE);
            part[si] += __shfl_xor(part[si], 32, WAVE);
        }
        float own[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const float x01 = lg & 1 ? part[4 + r] : part[r];
            const float x23 = lg & 1 ? part[12 + r] : part[8 + r];
            own[r] = lg * 4 + r <= lr ? (lg & 2 ? x23 : x01) : 0.f;
        }
#pragma unroll
        for (int j = 0; j < 4; ++j)
            if (j == w)
#pragma unroll
                for (int r = 0; r < 4; ++r) sc[j][r] = own[r] * k_scale;
    }
    // earlier sub-blocks (and a mild own one): q exp(L_t) against k exp(what lies
    // between s and the start of the own sub-block)
    {
        bf16x8_t qh[KK], ql[KK];
        float btw[KK][8];                                 // log decays of the sub-blocks between
#pragma unroll
        for (int kk = 0; kk < KK; ++kk)
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                __bf16 hi, lo;
                split_bf16_(qf[kk][e] * exp2_(lt[kk][e]), hi, lo);
                qh[kk][e] = hi; ql[kk][e] = lo;
                btw[kk][e] = 0.f;
            }
#pragma unroll
        for (int j = 3; j >= 0; --j) {
            if (j > w || (j == w && !mild)) continue;     // wave-uniform
            f32x4_t acc = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int kk = 0; kk < KK; ++kk) {
                const int d = kk * 32 + lg * 8;
                float kv[8], lv[8], tv8[8];
                load8<bf16>(reinterpret_cast<const bf16*>(kl) + (j * 16 + lr) * KS + d, kv);
                load8<float>(ll + (j * 16 + lr) * LS + d, lv);
                load8<float>(&tot[j][d], tv8);
                bf16x8_t kh, klo;
#pragma unroll
                for (int e = 0; e < 8; ++e) {
                    __bf16 hi, lo;
                    if (j < w) btw[kk][e] += tv8[e];      // now from the start of j to the start of w
                    split_bf16_(kv[e] * exp2_(btw[kk][e] - lv[e]), hi, lo);
                    kh[e] = hi; klo[e] = lo;
                }
                acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(klo, qh[kk], acc, 0, 0, 0);
                acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kh, ql[kk], acc, 0, 0, 0);
                acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kh, qh[kk], acc, 0, 0, 0);
            }
#pragma unroll
            for (int r = 0; r < 4; ++r)
                sc[j][r] = j < w || lg * 4 + r <= lr ? acc[r] * k_scale : 0.f;
        }
    }
    // ---- O += A V, two sub-blocks of keys at a time, A as hi + lo
#pragma unroll
    for (int pr = 0; pr < 2; ++pr) {
        if (pr * 2 > w) continue;                         // wave-uniform
        bf16x8_t ph, pl;
#pragma unroll
        for (int jj = 0; jj < 8; ++jj) {
            __bf16 hi, lo;
            split_bf16_(sc[pr * 2 + (jj >> 2)][jj & 3], hi, lo);
            ph[jj] = hi; pl[jj] = lo;
        }
#pragma unroll
        for (int nt = 0; nt < NT; ++nt) {
            union { bf16x8_t v; uint2 h2[2]; } vb;
            const uint16_t* vp = vt + (nt * 16 + lr) * GC_VS + pr * 32 + 4 * lg;
            vb.h2[0] = *reinterpret_cast<const uint2*>(vp);
            vb.h2[1] = *reinterpret_cast<const uint2*>(vp + 16);
            o[nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pl, vb.v, o[nt], 0, 0, 0);
            o[nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ph, vb.v, o[nt], 0, 0, 0);
        }
    }
    // ---- norm over the head's channels (tiles x 16 lanes), weight, silu gate
    float gw[4][NT];                                      // gates, loads in flight together
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        const bf16* gp = gate + (tok0 + min(w * 16 + lg * 4 + r, cnt - 1)) * gs + (long)h * Dv;
#pragma unroll
        for (int nt = 0; nt < NT; ++nt)
            gw[r][nt] = __bfloat162float(gp[min(nt * 16 + lr, Dv - 1)]);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        float ss = 0.f;
#pragma unroll
        for (int nt = 0; nt < NT; ++nt) ss += o[nt][r] * o[nt][r];   // channels past Dv are zero
        ss += __shfl_xor(ss, 1, WAVE);
        ss += __shfl_xor(ss, 2, WAVE);
        ss += __shfl_xor(ss, 4, WAVE);
        ss += __shfl_xor(ss, 8, WAVE);
        const int t = w * 16 + lg * 4 + r;
        if (t >= cnt) continue;
        const float inv = 1.f / sqrtf(ss / Dv + eps);
        bf16* op = out + (tok0 + t) * (long)(H * Dv) + (long)h * Dv;
#pragma unroll
        for (int nt = 0; nt < NT; ++nt) {
            const int nn = nt * 16 + lr;
            if (nn >= Dv) continue;
            const float gv = gw[r][nt];
            op[nn] = __float2bfloat16(o[nt][r] * inv * nw[nn] * (gv * sigmoidf_(gv)));
        }
    }
}

// ------------------------------------------------ grouped RMS norm with silu gate
// One wave per (row, group of C/groups channels): y (fp32) is multiplied by
// silu(gate) before the norm (gate_first) or after it; optional weight (C, or, wshared,
// C / groups for every group).
template <typename TG, typename TOut>
__global__ void group_gated_norm_kernel(const float* __restrict__ y, const TG* __restrict__ gate,
                                        long gs, const float* __restrict__ w, float eps,
                                        int groups, int gate_first, int wshared,
                                        TOut* __restrict__ out, long rows, int C) {
    const int lane = threadIdx.x & (WAVE - 1);
    const long id = (long)blockIdx.x * (blockDim.x / WAVE) + threadIdx.x / WAVE;
    if (id >= rows * groups) return;
    const long row = id / groups;
    const int gi = id % groups, Cg = C / groups;
    const float* yp = y + row * C + (long)gi * Cg;
    const TG* gp = gate + row * gs + (long)gi * Cg;
    const float* wp = w ? w + (wshared ? 0 : (long)gi * Cg) : nullptr;
    TOut* op = out + row * C + (long)gi * Cg;
    float ss = 0.f;
    for (int c = lane; c < Cg; c += WAVE) {
        float v = yp[c];
        if (gate_first) { const float gv = ldf<TG>(gp + c); v *= gv * sigmoidf_(gv); }
        ss += v * v;
    }
    const float inv = 1.f / sqrtf(wave_sum(ss) / Cg + eps);
    for (int c = lane; c < Cg; c += WAVE) {
        const float gv = ldf<TG>(gp + c);
        const float sg = gv * sigmoidf_(gv);
        float v = yp[c];
        if (gate_first) v *= sg;
        v *= inv;
        if (wp) v *= wp[c];
        if (!gate_first) v *= sg;
        stf<TOut>(op + c, v);
    }
}

// ------------------------------------------------------- group-limited router
// One wave per token: scores = softmax over E logits or their sigmoids (fp32), group
// score = best expert of the group or (gtwo) the sum of its two best, `keep` best
// groups stay, `top` best experts among them are chosen
// (ties: lowest index). Writes the dense (T, E + extra) weight row (zeros at
// unchosen experts, sigmoid gates in the extra columns), the chosen indices and
// their weights = score * scale (renormalised over the chosen first if asked, the
// sum plus norm_eps).
// `corr` (E, or null) is added to the scores for the group ranking and the choice
// only.
// A row whose logits are not numbers (the garbage of a pad token) selects the
// first experts with weight zero: every index stays in range.
DEV void wave_argmax(float& v, int& i) {
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
        const float ov = __shfl_xor(v, o, WAVE);
        const int oi = __shfl_xor(i, o, WAVE);
        if (ov > v || (ov == v && oi < i)) { v = ov; i = oi; }
    }
}

#define RT_WAVES 4
// one wave: logits `lp` (E + extra, global or LDS) of a token -> its dense row
// `dp`, chosen indices `idx` and weights `wts`; `cand` is 2E + ngroups floats of
// LDS scratch
DEV void route_select_(const float* lp, int E, int extra, int top, int ngroups, int keep,
                       float scale, int normalize, const float* __restrict__ corr, int sig,
                       int gtwo, float norm_eps, float* cand,
                       float* __restrict__ dp, int* __restrict__ idx, float* __restrict__ wts,
                       int lane) {
    float* gsc = cand + E;
    float* sco = gsc + ngroups;                   // the uncorrected scores (the weights)
    float rs = 1.f;
    if (sig) {                                    // uniform
        for (int e = lane; e < E; e += WAVE) cand[e] = sigmoidf_(lp[e]);
    } else {
        float m = -INFINITY;
        for (int e = lane; e < E; e += WAVE) m = fmaxf(m, lp[e]);
        m = wave_max(m);
        float sum = 0.f;
        for (int e = lane; e < E; e += WAVE) {
            const float x = expf(lp[e] - m);
            cand[e] = x;
            sum += x;
        }
        rs = 1.f / wave_sum(sum);
    }
    for (int e = lane; e < E; e += WAVE) {
        const float sc = cand[e] * rs;
        sco[e] = sc;
        cand[e] = corr ? sc + corr[e] : sc;       // the choice goes by the corrected score
        dp[e] = 0.f;
    }
    for (int x = lane; x < extra; x += WAVE) dp[E + x] = sigmoidf_(lp[E + x]);
    __builtin_amdgcn_wave_barrier();
    const int per = E / ngroups;
    if (ngroups > 1 && keep < ngroups) {
        for (int gi = lane; gi < ngroups; gi += WAVE) {
            float g1 = -INFINITY, g2 = -INFINITY;         // the two best of the group
            for (int j = 0; j < per; ++j) {
                const float x = cand[gi * per + j];
                g2 = fmaxf(g2, fminf(g1, x));
                g1 = fmaxf(g1, x);
            }
            gsc[gi] = gtwo && per > 1 ? g1 + g2 : g1;
        }
        __builtin_amdgcn_wave_barrier();
        for (int r = 0; r < keep; ++r) {
            float bv = -INFINITY; int bi = 0x7fffffff;
            for (int gi = lane; gi < ngroups; gi += WAVE) {
                const float x = gsc[gi];
                if (x < INFINITY && (x > bv)) { bv = x; bi = gi; }
            }
            wave_argmax(bv, bi);
            if ((unsigned)bi >= (unsigned)ngroups) bi = r;   // a row of NaNs compares false everywhere
            if (lane == 0) gsc[bi] = INFINITY;            // kept
            __builtin_amdgcn_wave_barrier();
        }
        for (int e = lane; e < E; e += WAVE) if (gsc[e / per] != INFINITY) cand[e] = -INFINITY;
        __builtin_amdgcn_wave_barrier();
    }
    float wsum = 0.f;
    float myw = 0.f; int myi = 0;                         // lane r keeps the r-th choice
    for (int r = 0; r < top; ++r) {
        float bv = -INFINITY; int bi = 0x7fffffff;
        for (int e = lane; e < E; e += WAVE) {
            const float x = cand[e];
            if (x > bv) { bv = x; bi = e; }
        }
        wave_argmax(bv, bi);
        if ((unsigned)bi >= (unsigned)E) { bi = r; bv = 0.f; }   // NaN row (a pad token): any valid index
        else bv = sco[bi];                                // the weight is the score itself
        if (lane == 0) cand[bi] = -INFINITY;
        if (lane == (r & (WAVE - 1))) {
            // more than 64 choices: flush the previous one first
            if (r >= WAVE) { idx[r - WAVE] = myi; wts[r - WAVE] = myw; }
            myw = bv; myi = bi;
        }
        wsum += bv;
        __builtin_amdgcn_wave_barrier();
    }
    const float f = normalize ? scale / (wsum + norm_eps) : scale;
    if (top <= WAVE) {
        if (lane < top) {
            idx[lane] = myi;
            wts[lane] = myw * f;
            dp[myi] = myw * f;
        }
    }
}

__global__ void __launch_bounds__(RT_WAVES * WAVE)
group_router_kernel(const float* __restrict__ logits, long ls, int E, int extra, int top,
                    int ngroups, int keep, float scale, int normalize,
                    const float* __restrict__ corr, int sig, int gtwo, float norm_eps,
                    float* __restrict__ dense, int* __restrict__ idx, float* __restrict__ wts,
                    long T) {
    extern __shared__ float rsm[];                // per wave: E choice scores + ngroups + E scores
    const int lane = threadIdx.x & (WAVE - 1), wv = threadIdx.x / WAVE;
    const long t = (long)blockIdx.x * RT_WAVES + wv;
    if (t >= T) return;
    route_select_(logits + t * ls, E, extra, top, ngroups, keep, scale, normalize, corr, sig,
                  gtwo, norm_eps, rsm + (long)wv * (2 * E + ngroups), dense + t * (long)(E + extra),
                  idx + t * top, wts + t * top, lane);
}

// Steps of few tokens: the router's product and its selection in one launch. One
// workgroup per token. The E + extra rows of the fp32 router weight are taken
// eight at a time: a thread reads its 8 channels of the token's input (widened to
// fp32) once and the same channels of the eight rows, all loads independent; the
// eight partial dot products are summed over the wave and over the four waves
// through LDS. The logits meet in LDS and the first wave selects as above.
template <typename T>
__global__ void __launch_bounds__(RT_WAVES * WAVE)
router_fused_kernel(const T* __restrict__ x, long xs, const float* __restrict__ w, int W, int vec,
                    int E, int extra, int top, int ngroups, int keep, float scale, int normalize,
                    const float* __restrict__ corr, const float* __restrict__ bias, int sig,
                    int gtwo, float norm_eps,
                    float* __restrict__ dense, int* __restrict__ idx, float* __restrict__ wts) {
    extern __shared__ float rsm[];                // E + extra logits, then the selection scratch
    __shared__ float part[RT_WAVES][8];
    const int tid = threadIdx.x, lane = tid & (WAVE - 1), wv = tid / WAVE;
    const long t = blockIdx.x;
    const T* xr = x + t * xs;
    const int rows = E + extra;
    for (int e0 = 0; e0 < rows; e0 += 8) {
        float acc[8];
#pragma unroll
        for (int k = 0; k < 8; ++k) acc[k] = 0.f;
        if (vec) {
            for (int c = tid * 8; c < W; c += RT_WAVES * WAVE * 8) {
                float xv[8];
                load8<T>(xr + c, xv);
                float wv8[8][8];                         // rows past the last repeat it
#pragma unroll
                for (int k = 0; k < 8; ++k)
                    load8<float>(w + (long)min(e0 + k, rows - 1) * W + c, wv8[k]);
#pragma unroll
                for (int k = 0; k < 8; ++k)
#pragma unroll
                    for (int j = 0; j < 8; ++j) acc[k] += xv[j] * wv8[k][j];
            }
        } else {
            for (int c = tid; c < W; c += RT_WAVES * WAVE) {
                const float xv = ldf<T>(xr + c);
#pragma unroll
                for (int k = 0; k < 8; ++k)
                    if (e0 + k < rows) acc[k] += xv * w[(long)(e0 + k) * W + c];
            }
        }
#pragma unroll
        for (int k = 0; k < 8; ++k) {
            const float v = wave_sum(acc[k]);
            if (lane == 0) part[wv][k] = v;
        }
        __syncthreads();
        if (tid < 8 && e0 + tid < rows) {
            float v = bias ? bias[e0 + tid] : 0.f;
#pragma unroll
            for (int q = 0; q < RT_WAVES; ++q) v += part[q][tid];
            rsm[e0 + tid] = v;
        }
        __syncthreads();
    }
    if (wv != 0) return;
    route_select_(rsm, E, extra, top, ngroups, keep, scale, normalize, corr, sig, gtwo,
                  norm_eps, rsm + E + extra,
                  dense + t * (long)(E + extra), idx + t * top, wts + t * top, lane);
}

// ------------------------------------------- activation times routing weight
// out[t, c] = act(x[t, c]) * gates[t, e], e = c / ff for an expert's columns (c <
// E*ff); the rest (a shared expert) takes gate column E, or one when there is no
// such column (gcols = E). gates = null: times one. act = relu^2 (0) or the exact
// gelu (1).
template <int ACT> DEV float expert_act_(float v) {
    if (ACT == 0) { const float r = fmaxf(v, 0.f); return r * r; }
    return 0.5f * v * (1.f + erff(v * 0.7071067811865476f));
}
DEV float expert_gate_(const float* __restrict__ gates, long t, int gcols, int c, int ff, int E) {
    const int e = min(c / ff, E);
    return (gates && e < gcols) ? gates[t * gcols + e] : 1.f;
}

template <typename T, int ACT>
__global__ void act_scale_kernel(const T* __restrict__ x, const float* __restrict__ gates,
                                 int gcols, int ff, int E, T* __restrict__ out, long rows, int C) {
    const long total = rows * C;
    for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < total;
         i += (long)gridDim.x * blockDim.x) {
        const long t = i / C;
        stf<T>(out + i, expert_act_<ACT>(ldf<T>(x + i)) *
                            expert_gate_(gates, t, gcols, i % C, ff, E));
    }
}

template <typename T, int ACT>
__global__ void act_scale_vec_kernel(const T* __restrict__ x, const float* __restrict__ gates,
                                     int gcols, int ff, int E, T* __restrict__ out, long rows,
                                     int C) {
    const int C8 = C / 8;
    const long total = rows * C8;
    for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < total;
         i += (long)gridDim.x * blockDim.x) {
        const long t = i / C8;
        const int c = (i % C8) * 8;
        const float gw = expert_gate_(gates, t, gcols, c, ff, E);
        float v[8];
        if (gw == 0.f) {                                  // an expert the token did not choose
#pragma unroll
            for (int e = 0; e < 8; ++e) v[e] = 0.f;
        } else {
            load8<T>(x + t * C + c, v);
#pragma unroll
            for (int e = 0; e < 8; ++e) v[e] = expert_act_<ACT>(v[e]) * gw;
        }
        store8<T>(out + t * C + c, v);
    }
}

// ----------------------------------------- gated units of stacked experts
// x (rows, 2C) = [gate | up] pre-activations of C = E*ff + shared columns.
// out[t, c] = glu(gate, up; limit) * gates[t, c / ff] for c < E*ff (an expert's
// columns, times the token's routing weight), glu(gate, up; shared_limit) for the
// rest (an always-on shared expert). ACT 0: glu = g sigmoid(alpha g) (u + 1) on the
// clamped pre-activations; ACT 1: glu = g sigmoid(g) u, no clamp.
template <int ACT> DEV float expert_glu_(float g, float u, float limit, float alpha) {
    return ACT == 0 ? clamped_glu_(g, u, limit, alpha) : g * sigmoidf_(g) * u;
}

template <typename T, int ACT>
__global__ void glu_scale_kernel(const T* __restrict__ x, const float* __restrict__ gates,
                                 long gs, int ff, int E, float limit, float slimit,
                                 float alpha, T* __restrict__ out, long rows, int C) {
    const long total = rows * C;
    const int ne = E * ff;
    for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < total;
         i += (long)gridDim.x * blockDim.x) {
        const long t = i / C;
        const int c = i % C;
        const bool own = c < ne;
        const float gw = own ? gates[t * gs + c / ff] : 1.f;
        float o = 0.f;
        if (gw != 0.f)
            o = expert_glu_<ACT>(ldf<T>(x + t * 2 * C + c), ldf<T>(x + t * 2 * C + C + c),
                                 own ? limit : slimit, alpha) * gw;
        stf<T>(out + i, o);
    }
}

template <typename T, int ACT>
__global__ void glu_scale_vec_kernel(const T* __restrict__ x,
                                     const float* __restrict__ gates, long gs, int ff,
                                     int E, float limit, float slimit, float alpha,
                                     T* __restrict__ out, long rows, int C) {
    const int C8 = C / 8;
    const long total = rows * C8;
    const int ne = E * ff;
    for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < total;
         i += (long)gridDim.x * blockDim.x) {
        const long t = i / C8;
        const int c = (i % C8) * 8;                      // ff % 8 == 0: one owner per 8 columns
        const bool own = c < ne;
        const float gw = own ? gates[t * gs + c / ff] : 1.f;
        float o[8];
        if (gw != 0.f) {                                 // an unchosen expert's columns are not read
            float g[8], u[8];
            load8<T>(x + t * 2 * C + c, g);
            load8<T>(x + t * 2 * C + C + c, u);
            const float lim = own ? limit : slimit;
#pragma unroll
            for (int e = 0; e < 8; ++e) o[e] = expert_glu_<ACT>(g[e], u[e], lim, alpha) * gw;
        } else {
#pragma unroll
            for (int e = 0; e < 8; ++e) o[e] = 0.f;
        }
        store8<T>(out + t * C + c, o);
    }
}

// y[t, c] *= sigmoid(gate[t, c]); gate rows may be a column slice (row stride gs)
template <typename T>
__global__ void sigmoid_gate_kernel(T* __restrict__ y, const T* __restrict__ gate, long gs,
                                    long rows, int C, int vec) {
    if (vec) {
        const int C8 = C / 8;
        const long total = rows * C8;
        for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < total;
             i += (long)gridDim.x * blockDim.x) {
            const long t = i / C8;
            const int c = (i % C8) * 8;
            float v[8], g[8];
            load8<T>(y + t * C + c, v);
            load8<T>(gate + t * gs + c, g);
#pragma unroll
            for (int e = 0; e < 8; ++e) v[e] *= sigmoidf_(g[e]);
            store8<T>(y + t * C + c, v);
        }
        return;
    }
    const long total = rows * C;
    for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < total;
         i += (long)gridDim.x * blockDim.x) {
        const long t = i / C;
        const int c = i % C;
        stf<T>(y + i, ldf<T>(y + i) * sigmoidf_(ldf<T>(gate + t * gs + c)));
    }
}

// 16-byte variant for rows of up to LN_THREADS * 8 * NV channels: every term is
// read once and stays in registers between the statistics and the update
template <typename T, int NV>
__global__ void __launch_bounds__(LN_THREADS)
scaled_residual_vec_kernel(float* __restrict__ x, const T* __restrict__ y0,
                           const float* __restrict__ w0, int n0, const T* __restrict__ y1,
                           const float* __restrict__ w1, int n1, const T* __restrict__ y2,
                           const float* __restrict__ w2, int n2, float eps, int C) {
    __shared__ float red[3][LN_THREADS / WAVE];
    const long row = blockIdx.x;
    const T* ys[3] = {y0, y1, y2};
    const float* ws[3] = {w0, w1, w2};
    const int ns[3] = {n0, n1, n2};
    float val[3][NV][8];
    float ss[3] = {0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < 3; ++i) {
        if (!ys[i]) continue;                             // uniform
#pragma unroll
        for (int j = 0; j < NV; ++j) {
            const int c = (j * LN_THREADS + threadIdx.x) * 8;
            if (c < C) {
                load8<T>(ys[i] + row * C + c, val[i][j]);
#pragma unroll
                for (int e = 0; e < 8; ++e) ss[i] += val[i][j][e] * val[i][j][e];
            }
        }
    }
    const int lane = threadIdx.x & (WAVE - 1), wv = threadIdx.x / WAVE;
#pragma unroll
    for (int i = 0; i < 3; ++i) {
        const float t = wave_sum(ss[i]);
        if (lane == 0) red[i][wv] = t;
    }
    __syncthreads();
    float inv[3];
#pragma unroll
    for (int i = 0; i < 3; ++i) {
        float t = 0.f;
#pragma unroll
        for (int k = 0; k < LN_THREADS / WAVE; ++k) t += red[i][k];
        inv[i] = (ys[i] && ns[i]) ? 1.f / sqrtf(t / C + eps) : 1.f;
    }
#pragma unroll
    for (int j = 0; j < NV; ++j) {
        const int c = (j * LN_THREADS + threadIdx.x) * 8;
        if (c >= C) continue;
        float xv[8];
        load8<float>(x + row * C + c, xv);
#pragma unroll
        for (int i = 0; i < 3; ++i) {
            if (!ys[i]) continue;
            float wv8[8];
            load8<float>(ws[i] + c, wv8);
#pragma unroll
            for (int e = 0; e < 8; ++e) xv[e] += val[i][j][e] * inv[i] * wv8[e];
        }
        st8<float>(x + row * C + c, xv);
    }
}

// ------------------------------------------- embedding + learned position rows
// stream[t, :] = float(emb[t, :]) + float(table[max(pos[t], 0), :])
template <typename T>
__global__ void embed_pos_kernel(const T* __restrict__ emb, const T* __restrict__ table,
                                 const int* __restrict__ pos, float* __restrict__ out,
                                 long ntok, int C, int rows_in_table) {
    const long total = ntok * C;
    for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < total;
         i += (long)gridDim.x * blockDim.x) {
        const long t = i / C;
        const int c = i % C;
        int p = pos[t];
        p = p < 0 ? 0 : (p >= rows_in_table ? rows_in_table - 1 : p);
        out[i] = ldf<T>(emb + i) + ldf<T>(table + (long)p * C + c);
    }
}

// ------------------------------------------------ token + bigram embedding rows
// stream[t, :] = emb[tok] + table[row], row = (prev * mul_prev + tok * mul_cur) mod
// buckets, or `buckets` (the last row) at position 0. `prev` is the token before it in
// the row; for a row's first column it is carried per state slot in `last`, which the
// workgroup of that column (its only reader) then sets to the row's last real token.
// One workgroup per token; pad tokens give zero rows.
template <typename T>
__global__ void __launch_bounds__(256)
bigram_embed_kernel(const long long* __restrict__ ids, const int* __restrict__ pos,
                    const int* __restrict__ seq, const int* __restrict__ nvalid,
                    const T* __restrict__ emb, const T* __restrict__ table,
                    int* __restrict__ last, long long mul_prev, long long mul_cur,
                    long long buckets, int vocab, float* __restrict__ out, int S, int C, int vec) {
    const long tok = blockIdx.x;
    const int b = tok / S, t = tok % S, slot = seq[b], p = pos[tok];
    float* op = out + tok * C;
    if (p < 0 || slot < 0) {                              // uniform
        for (int c = threadIdx.x; c < C; c += 256) op[c] = 0.f;
        return;
    }
    const long long cur = min(max(ids[tok], 0ll), (long long)vocab - 1);
    long long row = buckets;
    if (p > 0) {
        const long long prev = t > 0 ? ids[tok - 1] : (long long)last[slot];
        row = (prev * mul_prev + cur * mul_cur) % buckets;
        if (row < 0) row += buckets;
    }
    if (t == 0) {
        __syncthreads();                                  // `last` has been read
        if (threadIdx.x == 0) last[slot] = (int)ids[tok + nvalid[b] - 1];
    }
    const T* ep = emb + cur * C;
    const T* tp = table + row * C;
    if (vec) {
        for (int c = threadIdx.x * 8; c < C; c += 256 * 8) {
            float a[8], g[8];
            load8<T>(ep + c, a);
            load8<T>(tp + c, g);
#pragma unroll
            for (int e = 0; e < 8; ++e) a[e] += g[e];
            st8<float>(op + c, a);
        }
    } else {
        for (int c = threadIdx.x; c < C; c += 256) op[c] = ldf<T>(ep + c) + ldf<T>(tp + c);
    }
}

// -------------------------------------------------- per-layer token input, gated
// out[t, c] = gelu_tanh(z[t, c]) * table[tok, off + c]: a layer's slice of the token's
// row in a (vocab, layers * C) table, gated by a projection of the stream
template <typename T>
__global__ void token_gate_kernel(const T* __restrict__ z, long zs,
                                  const long long* __restrict__ ids, const T* __restrict__ table,
                                  long ts, int off, int vocab, T* __restrict__ out, long rows,
                                  int C) {
    const long total = rows * C;
    for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < total;
         i += (long)gridDim.x * blockDim.x) {
        const long t = i / C;
        const int c = i % C;
        const long long tok = min(max(ids[t], 0ll), (long long)vocab - 1);
        stf<T>(out + i, gelu_tanh_(ldf<T>(z + t * zs + c)) * ldf<T>(table + tok * ts + off + c));
    }
}

// The same with the gating projection z = h . wg^T inside: workgroup = 16 tokens x
// 16 channels on the matrix cores, the product's inner dimension split over 8 waves
// and summed through LDS.
__global__ void __launch_bounds__(512)
token_gate_proj_kernel(const bf16* __restrict__ x, long xs, const bf16* __restrict__ wg, int K,
                       const long long* __restrict__ ids, const bf16* __restrict__ table, long ts,
                       int off, int vocab, bf16* __restrict__ out, long rows, int C) {
    __shared__ float red[8][256];
    const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
    const int lr = lane & 15, lg = lane >> 4;
    const long t0 = (long)blockIdx.y * 16;
    const int n0 = blockIdx.x * 16;
    const bool tok = t0 + lr < rows, ch = n0 + lr < C;
    const bf16* xp = x + (tok ? t0 + lr : 0) * xs + lg * 8;
    const bf16* wp = wg + (long)(ch ? n0 + lr : 0) * K + lg * 8;
    f32x4_t acc = f32x4_t{0.f, 0.f, 0.f, 0.f};
    for (int k0 = wv * 32; k0 < K; k0 += 8 * 32) {
        uint4 xa = make_uint4(0, 0, 0, 0), wa = make_uint4(0, 0, 0, 0);
        if (k0 + lg * 8 < K) {
            if (tok) xa = *reinterpret_cast<const uint4*>(xp + k0);
            if (ch) wa = *reinterpret_cast<const uint4*>(wp + k0);
        }
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
            __builtin_bit_cast(bf16x8_t, xa), __builtin_bit_cast(bf16x8_t, wa), acc, 0, 0, 0);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) red[wv][(lg * 4 + r) * 16 + lr] = acc[r];
    __syncthreads();
    if (tid < 256) {
        const long t = t0 + tid / 16;
        const int n = n0 + tid % 16;
        if (t < rows && n < C) {
            float z = 0.f;
#pragma unroll
            for (int i = 0; i < 8; ++i) z += red[i][tid];
            const long long id = min(max(ids[t], 0ll), (long long)vocab - 1);
            out[t * C + n] = __float2bfloat16(
                gelu_tanh_(z) * __bfloat162float(table[id * ts + off + n]));
        }
    }
}

// ------------------------------------------------ one product per head, few tokens
// out[t, h, n] = sum_k a[t, h, k] w[h, n, k] (both operands contiguous over k).
// Workgroup = 16 output channels of a head x 64 tokens; its 4 waves split k and sum
// through LDS, so every weight row is fetched once.
__global__ void __launch_bounds__(256)
head_product_kernel(const bf16* __restrict__ a, const bf16* __restrict__ w,
                    bf16* __restrict__ out, int T, int H, int K, int N) {
    __shared__ float red[4][4][256];
    const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
    const int lr = lane & 15, lg = lane >> 4;
    const int n0 = blockIdx.x * 16, h = blockIdx.y, t0 = blockIdx.z * 64;
    const bool ch = n0 + lr < N;
    const bf16* wp = w + ((long)h * N + (ch ? n0 + lr : 0)) * K + lg * 8;
    f32x4_t acc[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) acc[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int k0 = wv * 32; k0 < K; k0 += 4 * 32) {
        const bool kin = k0 + lg * 8 < K;
        uint4 wa = make_uint4(0, 0, 0, 0);
        if (kin && ch) wa = *reinterpret_cast<const uint4*>(wp + k0);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int t = t0 + i * 16 + lr;
            uint4 av = make_uint4(0, 0, 0, 0);
            if (kin && t < T)
                av = *reinterpret_cast<const uint4*>(a + ((long)t * H + h) * K + k0 + lg * 8);
            acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                __builtin_bit_cast(bf16x8_t, av), __builtin_bit_cast(bf16x8_t, wa), acc[i], 0, 0, 0);
        }
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) red[wv][i][(lg * 4 + r) * 16 + lr] = acc[i][r];
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int t = t0 + i * 16 + tid / 16, n = n0 + tid % 16;
        if (t < T && n < N)
            out[((long)t * H + h) * N + n] = __float2bfloat16(
                red[0][i][tid] + red[1][i][tid] + red[2][i][tid] + red[3][i][tid]);
    }
}

// ------------------------------------- residual sum of weighted, optionally normed terms
// x[row] += sum_i f_i(y_i[row]) * w_i, f_i = RMS norm over the row or identity.
// One workgroup per row; statistics fp32.
template <typename T>
__global__ void __launch_bounds__(LN_THREADS)
scaled_residual_kernel(float* __restrict__ x, const T* __restrict__ y0,
                       const float* __restrict__ w0, int n0, const T* __restrict__ y1,
                       const float* __restrict__ w1, int n1, const T* __restrict__ y2,
                       const float* __restrict__ w2, int n2, float eps, int C) {
    __shared__ float red[LN_THREADS / WAVE];
    const long row = blockIdx.x;
    const T* ys[3] = {y0, y1, y2};
    const float* ws[3] = {w0, w1, w2};
    const int ns[3] = {n0, n1, n2};
    float inv[3] = {1.f, 1.f, 1.f};
    float ss[3] = {0.f, 0.f, 0.f};
    for (int c = threadIdx.x; c < C; c += LN_THREADS) {
#pragma unroll
        for (int i = 0; i < 3; ++i)
            if (ys[i] && ns[i]) { const float v = ldf<T>(ys[i] + row * C + c); ss[i] += v * v; }
    }
#pragma unroll
    for (int i = 0; i < 3; ++i)
        if (ys[i] && ns[i]) inv[i] = 1.f / sqrtf(block_sum(ss[i], red) / C + eps);   // uniform
    float* xr = x + row * C;
    for (int c = threadIdx.x; c < C; c += LN_THREADS) {
        float acc = 0.f;
#pragma unroll
        for (int i = 0; i < 3; ++i)
            if (ys[i]) acc += ldf<T>(ys[i] + row * C + c) * inv[i] * ws[i][c];
        xr[c] += acc;
    }
}

// =================================================================== C ABI
// ------------------------------------------------- parallel residual streams
// A token's residual is NS streams of C channels (fp32). One step: every stream anew
// from the old ones, x_t = sum_s mix[s, t] x_s + wout[t] * y (y null: the streams are
// only read), then u = sum_t win[t] x_t (win null: their plain sum) and, with nw, its
// layer norm (mean, variance of the deviations, weight, no bias) in the next GEMM's
// type, else u itself in fp32. `xstr` is the distance between a token's streams in
// `xin`; 0 reads one row for all of them (streams that still equal the embedding).
// One workgroup per token. The vector form reads and writes each operand once (new
// streams go straight out, u stays in registers) and may run in place.
template <typename T, int NS, int NV>
__global__ void __launch_bounds__(LN_THREADS)
hyper_step_vec_kernel(const float* xin, long xrow, long xstr, const T* __restrict__ y,
                      const float* __restrict__ mix, const float* __restrict__ wout, float* xout,
                      const float* __restrict__ win, const float* __restrict__ nw, float eps,
                      T* __restrict__ hout, float* __restrict__ uout, int C) {
    __shared__ float red[LN_THREADS / WAVE];
    const long row = blockIdx.x;
    float wi[NS];
#pragma unroll
    for (int t = 0; t < NS; ++t) wi[t] = win ? win[t] : 1.f;
    float u[NV][4];
    float sum = 0.f;
#pragma unroll
    for (int j = 0; j < NV; ++j) {
        const int c = (j * LN_THREADS + threadIdx.x) * 4;
#pragma unroll
        for (int e = 0; e < 4; ++e) u[j][e] = 0.f;
        if (c >= C) continue;
        float x[NS][4], yv[4];
#pragma unroll
        for (int s = 0; s < NS; ++s) {
            const float4 v = *reinterpret_cast<const float4*>(xin + row * xrow + s * xstr + c);
            x[s][0] = v.x; x[s][1] = v.y; x[s][2] = v.z; x[s][3] = v.w;
        }
        if (y) {
            load4<T>(y + row * C + c, yv);
#pragma unroll
            for (int t = 0; t < NS; ++t) {
                float o[4];
                const float wo = wout[t];
#pragma unroll
                for (int e = 0; e < 4; ++e) o[e] = wo * yv[e];
#pragma unroll
                for (int s = 0; s < NS; ++s) {
                    const float m = mix[s * NS + t];
#pragma unroll
                    for (int e = 0; e < 4; ++e) o[e] += m * x[s][e];
                }
                if (xout)
                    *reinterpret_cast<float4*>(xout + (row * NS + t) * (long)C + c) =
                        make_float4(o[0], o[1], o[2], o[3]);
#pragma unroll
                for (int e = 0; e < 4; ++e) u[j][e] += wi[t] * o[e];
            }
        } else {
#pragma unroll
            for (int t = 0; t < NS; ++t)
#pragma unroll
                for (int e = 0; e < 4; ++e) u[j][e] += wi[t] * x[t][e];
        }
        if (!nw)
            *reinterpret_cast<float4*>(uout + row * C + c) =
                make_float4(u[j][0], u[j][1], u[j][2], u[j][3]);
        sum += u[j][0] + u[j][1] + u[j][2] + u[j][3];
    }
    if (!nw) return;                                      // uniform
    const float mean = block_sum(sum, red) / C;
    float q = 0.f;
#pragma unroll
    for (int j = 0; j < NV; ++j)
        if ((j * LN_THREADS + threadIdx.x) * 4 < C)
#pragma unroll
            for (int e = 0; e < 4; ++e) { u[j][e] -= mean; q += u[j][e] * u[j][e]; }
    const float inv = 1.f / sqrtf(block_sum(q, red) / C + eps);
#pragma unroll
    for (int j = 0; j < NV; ++j) {
        const int c = (j * LN_THREADS + threadIdx.x) * 4;
        if (c >= C) continue;
        const float4 w4 = *reinterpret_cast<const float4*>(nw + c);
        const float o[4] = {u[j][0] * inv * w4.x, u[j][1] * inv * w4.y, u[j][2] * inv * w4.z,
                            u[j][3] * inv * w4.w};
        store4<T>(hout + row * C + c, o);
    }
}

// scalar form: any number of streams, width and alignment; not in place
template <typename T>
__global__ void __launch_bounds__(LN_THREADS)
hyper_step_kernel(const float* __restrict__ xin, long xrow, long xstr, const T* __restrict__ y,
                  const float* __restrict__ mix, const float* __restrict__ wout,
                  float* __restrict__ xout, const float* __restrict__ win,
                  const float* __restrict__ nw, float eps, T* __restrict__ hout,
                  float* __restrict__ uout, float* __restrict__ scratch, int NS, int C) {
    __shared__ float red[LN_THREADS / WAVE];
    const long row = blockIdx.x;
    const float* xr = xin + row * xrow;
    float* ur = (nw ? scratch : uout) + row * C;          // re-read by the same thread only
    float sum = 0.f;
    for (int c = threadIdx.x; c < C; c += LN_THREADS) {
        float u = 0.f;
        const float yv = y ? ldf<T>(y + row * C + c) : 0.f;
        for (int t = 0; t < NS; ++t) {
            float o;
            if (y) {
                o = wout[t] * yv;
                for (int s = 0; s < NS; ++s) o += mix[s * NS + t] * xr[s * xstr + c];
                if (xout) xout[(row * NS + t) * (long)C + c] = o;
            } else {
                o = xr[t * xstr + c];
            }
            u += (win ? win[t] : 1.f) * o;
        }
        ur[c] = u;
        sum += u;
    }
    if (!nw) return;                                      // uniform
    const float mean = block_sum(sum, red) / C;
    float q = 0.f;
    for (int c = threadIdx.x; c < C; c += LN_THREADS) { const float d = ur[c] - mean; q += d * d; }
    const float inv = 1.f / sqrtf(block_sum(q, red) / C + eps);
    for (int c = threadIdx.x; c < C; c += LN_THREADS)
        stf<T>(hout + row * C + c, (ur[c] - mean) * inv * nw[c]);
}

// ------------------------------------- attention rows of a step in one launch
// Queries and keys of a token: rotary positions (half-split pairs i, i + half of the
// first 2*half channels, fp32 angle pos * inv_freq[i]; half = 0: none), then (unorm)
// divided by the head's root mean square over D; queries go to a dense buffer, keys
// into the token's page slot. Values, optionally mixed with another layer's values of
// the same token, v' = (1 - lam) v + lam v_first (fp32), go into the page slot as they
// come. One workgroup per token: the angles' cosines and sines are made once for all
// heads. Pad tokens get zero queries and write no page.
template <typename T>
__global__ void __launch_bounds__(256)
qkv_rows_vec_kernel(const T* __restrict__ q, long qs, const T* __restrict__ k, long ks,
                    const T* __restrict__ v, long vs, const T* __restrict__ vf, long vfs,
                    const float* __restrict__ lam, const int* __restrict__ pos,
                    const int* __restrict__ slots, const float* __restrict__ inv_freq, int half,
                    int unorm, float eps, T* __restrict__ qo, T* __restrict__ kc,
                    T* __restrict__ vc, long nslots, int H, int G, int D, int Dv, int lanes) {
    __shared__ __attribute__((aligned(16))) float cs[HN_MAXC / 2], sn[HN_MAXC / 2];
    const long tok = blockIdx.x;
    const int tid = threadIdx.x;
    const int p = pos[tok];
    if (p < 0) {
        const float z[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
        for (int c = tid * 8; c < H * D; c += 256 * 8) store8<T>(qo + tok * H * D + c, z);
        return;
    }
    for (int i = tid; i < half; i += 256) {
        float s_, c_;
        sincosf((float)p * inv_freq[i], &s_, &c_);
        cs[i] = c_;
        sn[i] = s_;
    }
    const long slot = slots[tok];
    const bool wr = slot >= 0 && slot < nslots;
    if (wr) {
        const float l = vf ? *lam : 0.f;
        for (int c = tid * 8; c < G * Dv; c += 256 * 8) {
            float x[8];
            load8<T>(v + tok * vs + c, x);
            if (vf) {
                float f[8];
                load8<T>(vf + tok * vfs + c, f);
#pragma unroll
                for (int e = 0; e < 8; ++e) x[e] = (1.f - l) * x[e] + l * f[e];
            }
            store8<T>(vc + slot * (long)(G * Dv) + c, x);
        }
    }
    __syncthreads();
    // `lanes` (a power of two, at most a wave) neighbours share a head, 8 channels each
    const int li = tid % lanes, c = li * 8;
    for (int u = tid / lanes; u < H + G; u += 256 / lanes) {
        const bool isq = u < H;
        const T* xp = isq ? q + tok * qs + (long)u * D : k + tok * ks + (long)(u - H) * D;
        float x[8];
        float ss = 0.f;
        const bool ok = c < D;
        if (ok) {
            load8<T>(xp + c, x);
#pragma unroll
            for (int e = 0; e < 8; ++e) ss += x[e] * x[e];
        }
        float inv = 1.f;                                  // rotation leaves the norm as it is
        if (unorm) {
            for (int o = lanes / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, WAVE);
            inv = 1.f / sqrtf(ss / D + eps);
        }
        if (!ok) continue;
        if (c < 2 * half) {
            const bool lo = c < half;
            const int a = lo ? c : c - half;
            float w[8], cv[8], sv[8];
            load8<T>(xp + (lo ? c + half : a), w);        // the partner channels
            load8<float>(cs + a, cv);
            load8<float>(sn + a, sv);
#pragma unroll
            for (int e = 0; e < 8; ++e)
                x[e] = lo ? x[e] * cv[e] - w[e] * sv[e] : x[e] * cv[e] + w[e] * sv[e];
        }
#pragma unroll
        for (int e = 0; e < 8; ++e) x[e] *= inv;
        if (isq) store8<T>(qo + (tok * H + u) * (long)D + c, x);
        else if (wr) store8<T>(kc + (slot * G + (u - H)) * (long)D + c, x);
    }
}

// scalar form: any sizes and alignment; a wave per head
template <typename T>
__global__ void __launch_bounds__(256)
qkv_rows_kernel(const T* __restrict__ q, long qs, const T* __restrict__ k, long ks,
                const T* __restrict__ v, long vs, const T* __restrict__ vf, long vfs,
                const float* __restrict__ lam, const int* __restrict__ pos,
                const int* __restrict__ slots, const float* __restrict__ inv_freq, int half,
                int unorm, float eps, T* __restrict__ qo, T* __restrict__ kc,
                T* __restrict__ vc, long nslots, int H, int G, int D, int Dv) {
    __shared__ float cs[HN_MAXC / 2], sn[HN_MAXC / 2];
    const long tok = blockIdx.x;
    const int tid = threadIdx.x, lane = tid & (WAVE - 1), wv = tid / WAVE;
    const int p = pos[tok];
    if (p < 0) {
        for (int c = tid; c < H * D; c += 256) stf<T>(qo + tok * H * D + c, 0.f);
        return;
    }
    for (int i = tid; i < half; i += 256) {
        float s_, c_;
        sincosf((float)p * inv_freq[i], &s_, &c_);
        cs[i] = c_;
        sn[i] = s_;
    }
    const long slot = slots[tok];
    const bool wr = slot >= 0 && slot < nslots;
    if (wr) {
        const float l = vf ? *lam : 0.f;
        for (int c = tid; c < G * Dv; c += 256) {
            float x = ldf<T>(v + tok * vs + c);
            if (vf) x = (1.f - l) * x + l * ldf<T>(vf + tok * vfs + c);
            stf<T>(vc + slot * (long)(G * Dv) + c, x);
        }
    }
    __syncthreads();
    for (int u = wv; u < H + G; u += 4) {
        const bool isq = u < H;
        const T* xp = isq ? q + tok * qs + (long)u * D : k + tok * ks + (long)(u - H) * D;
        T* op = isq ? qo + (tok * H + u) * (long)D
                    : (wr ? kc + (slot * G + (u - H)) * (long)D : nullptr);
        float inv = 1.f;
        if (unorm) {
            float ss = 0.f;
            for (int c = lane; c < D; c += WAVE) { const float x = ldf<T>(xp + c); ss += x * x; }
            inv = 1.f / sqrtf(wave_sum(ss) / D + eps);
        }
        if (!op) continue;                                // wave-uniform
        for (int i = lane; i < half; i += WAVE) {
            const float a = ldf<T>(xp + i), b = ldf<T>(xp + i + half);
            stf<T>(op + i, (a * cs[i] - b * sn[i]) * inv);
            stf<T>(op + i + half, (b * cs[i] + a * sn[i]) * inv);
        }
        for (int c = 2 * half + lane; c < D; c += WAVE) stf<T>(op + c, ldf<T>(xp + c) * inv);
    }
}

// -------------------------------------- matrix memory with exponential gates
// Per head: log input gate i = cap tanh(z_i / cap), log forget gate f = log sigmoid(cap
// tanh(z_f / cap)) (z with their fp32 biases), running maximum m_t = max(f + m_{t-1}, i)
// from m = 0; S_t = a_t S_{t-1} + w_t k v^T and n_t likewise with k alone, a_t = exp(f +
// m_{t-1} - m_t), w_t = exp(i - m_t), o = S^T q / (max(|n.q|, exp(-m)) + 1e-6). The
// state of a head is (Dv + 1) rows of D key channels: a row per value channel, then n
// (the row of a value channel that is always one). Both exponents are never positive.
DEV void mlstm_gate_(float zi, float zf, float cap, float& i, float& f) {
    const float x = cap * tanhf(zf / cap);
    i = cap * tanhf(zi / cap);
    f = fminf(x, 0.f) - log1pf(expf(-fabsf(x)));
}

#define MG_THREADS 512
#define MG_KEEP 8
// One workgroup per (row, head): log a, w and m of every token of the step, and the
// carried m. A thread owns consecutive tokens; (sum of f, running maximum from minus
// infinity) pairs of the threads' spans are combined by a scan, then every thread
// walks its span from its true start. Spans of up to MG_KEEP tokens keep their gates
// in registers, longer ones make them again.
template <typename T>
__global__ void __launch_bounds__(MG_THREADS)
mlstm_gates_kernel(const T* __restrict__ zi, long zis, const T* __restrict__ zf, long zfs,
                   const float* __restrict__ bi, const float* __restrict__ bf, float cap,
                   float* __restrict__ mstate, const int* __restrict__ pos,
                   const int* __restrict__ seq, const int* __restrict__ nvalid,
                   float* __restrict__ ld, float* __restrict__ wt, float* __restrict__ mx,
                   int S, int H) {
    __shared__ float wf[MG_THREADS / WAVE], wm[MG_THREADS / WAVE];
    const int h = blockIdx.x, b = blockIdx.y;
    const int slot = seq[b], n = slot < 0 ? 0 : nvalid[b];
    if (n <= 0) return;                                   // uniform
    const int tid = threadIdx.x, lane = tid & (WAVE - 1), wv = tid / WAVE;
    const int per = (n + MG_THREADS - 1) / MG_THREADS;
    const int t0 = min(n, tid * per), t1 = min(n, t0 + per);
    const float bih = bi[h], bfh = bf[h];
    const long tok0 = (long)b * S;
    float F = 0.f, M = -INFINITY;
    float ik[MG_KEEP], fk[MG_KEEP];
    const bool kept_all = per <= MG_KEEP;                 // uniform
    if (kept_all) {
#pragma unroll
        for (int x = 0; x < MG_KEEP; ++x) {               // loads in flight together
            const long tk = tok0 + min(t0 + x, n - 1);
            ik[x] = ldf<T>(zi + tk * zis + h) + bih;
            fk[x] = ldf<T>(zf + tk * zfs + h) + bfh;
        }
#pragma unroll
        for (int x = 0; x < MG_KEEP; ++x) {
            if (x >= t1 - t0) continue;
            mlstm_gate_(ik[x], fk[x], cap, ik[x], fk[x]);
            F += fk[x];
            M = fmaxf(M + fk[x], ik[x]);
        }
    } else {
        for (int t = t0; t < t1; ++t) {
            float i, f;
            mlstm_gate_(ldf<T>(zi + (tok0 + t) * zis + h) + bih,
                        ldf<T>(zf + (tok0 + t) * zfs + h) + bfh, cap, i, f);
            F += f;
            M = fmaxf(M + f, i);
        }
    }
    float pf = F, pm = M;                                 // inclusive over the wave
#pragma unroll
    for (int o = 1; o < WAVE; o <<= 1) {
        const float of = __shfl_up(pf, o, WAVE), om = __shfl_up(pm, o, WAVE);
        if (lane >= o) { pm = fmaxf(om + pf, pm); pf += of; }
    }
    if (lane == WAVE - 1) { wf[wv] = pf; wm[wv] = pm; }
    __syncthreads();
    float m = pos[tok0] > 0 ? mstate[(long)slot * H + h] : 0.f;
    for (int x = 0; x < wv; ++x) m = fmaxf(m + wf[x], wm[x]);
    const float ef = __shfl_up(pf, 1, WAVE), em = __shfl_up(pm, 1, WAVE);
    if (lane > 0) m = fmaxf(m + ef, em);
    auto step = [&](int t, float i, float f) {
        const float kept = f + m;
        m = fmaxf(kept, i);
        const long at = (tok0 + t) * H + h;
        ld[at] = kept - m;
        wt[at] = expf(i - m);
        mx[at] = m;
    };
    if (kept_all) {
#pragma unroll
        for (int x = 0; x < MG_KEEP; ++x)
            if (x < t1 - t0) step(t0 + x, ik[x], fk[x]);
    } else {
        for (int t = t0; t < t1; ++t) {
            float i, f;
            mlstm_gate_(ldf<T>(zi + (tok0 + t) * zis + h) + bih,
                        ldf<T>(zf + (tok0 + t) * zfs + h) + bfh, cap, i, f);
            step(t, i, f);
        }
    }
    __syncthreads();                                      // every thread has read the carried m
    if (t1 == n && t0 < n) mstate[(long)slot * H + h] = m;
}

// Read-out of the scan's rows o (rows, H, Dv + 1) fp32: a wave per (token, head)
// divides by the normalizer, then by the head's root mean square, times the weight
// (H * Dv) and the sigmoid of the gate.
template <typename T>
__global__ void mlstm_readout_kernel(const float* __restrict__ o, const float* __restrict__ mx,
                                     const T* __restrict__ gate, long gs,
                                     const float* __restrict__ nw, float eps,
                                     const int* __restrict__ pos, T* __restrict__ out, long rows,
                                     int H, int Dv) {
    const int lane = threadIdx.x & (WAVE - 1);
    const long id = (long)blockIdx.x * (blockDim.x / WAVE) + threadIdx.x / WAVE;
    if (id >= rows * H) return;
    const long row = id / H;
    const int h = id % H;
    T* op = out + row * (long)H * Dv + (long)h * Dv;
    if (pos[row] < 0) {
        for (int c = lane; c < Dv; c += WAVE) stf<T>(op + c, 0.f);
        return;
    }
    const float* rp = o + id * (Dv + 1);
    const float inv = 1.f / (fmaxf(fabsf(rp[Dv]), expf(-mx[id])) + 1e-6f);
    float ss = 0.f;
    for (int c = lane; c < Dv; c += WAVE) { const float x = rp[c] * inv; ss += x * x; }
    const float nrm = inv / sqrtf(wave_sum(ss) / Dv + eps);
    const T* gp = gate + row * gs + (long)h * Dv;
    for (int c = lane; c < Dv; c += WAVE)
        stf<T>(op + c, rp[c] * nrm * nw[h * Dv + c] * sigmoidf_(ldf<T>(gp + c)));
}

#define MD_THREADS 512
// Single-token steps in one launch: gates, state update, read-out, norm and gate of a
// (row, head). `lanes` (a power of two, at most a wave) neighbours share a state row;
// with `vec` each of them holds four consecutive channels, else the channels lane,
// lane + lanes, ... (at most four).
template <typename T>
__global__ void __launch_bounds__(MD_THREADS)
mlstm_decode_kernel(const T* __restrict__ q, long qs, const T* __restrict__ k, long ks,
                    const T* __restrict__ v, long vs, const T* __restrict__ zi, long zis,
                    const T* __restrict__ zf, long zfs, const float* __restrict__ bi,
                    const float* __restrict__ bf, float cap, float k_scale,
                    const T* __restrict__ gate, long gs, const float* __restrict__ nw, float eps,
                    float* __restrict__ state, float* __restrict__ mstate,
                    const int* __restrict__ pos, const int* __restrict__ seq,
                    T* __restrict__ out, int H, int D, int Dv, int lanes, int vec) {
    extern __shared__ float osm[];                        // Dv + 1 read-outs
    __shared__ float red[MD_THREADS / WAVE];
    const int h = blockIdx.x, b = blockIdx.y, tid = threadIdx.x;
    const int slot = seq[b], p = pos[b];
    T* op = out + ((long)b * H + h) * Dv;
    if (slot < 0 || p < 0) {                              // uniform
        for (int c = tid; c < Dv; c += MD_THREADS) stf<T>(op + c, 0.f);
        return;
    }
    float i, f;
    mlstm_gate_(ldf<T>(zi + b * zis + h) + bi[h], ldf<T>(zf + b * zfs + h) + bf[h], cap, i, f);
    float m = p > 0 ? mstate[(long)slot * H + h] : 0.f;
    const float kept = f + m;
    m = fmaxf(kept, i);
    const float a = p > 0 ? expf(kept - m) : 0.f, w = expf(i - m);
    const int li = tid % lanes;
    float kr[4], qr[4];
    int dd[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        dd[e] = vec ? li * 4 + e : li + e * lanes;
        const bool ok = dd[e] < D;
        kr[e] = ok ? ldf<T>(k + b * ks + (long)h * D + dd[e]) * k_scale * w : 0.f;
        qr[e] = ok ? ldf<T>(q + b * qs + (long)h * D + dd[e]) : 0.f;
    }
    float* sp = state + ((long)slot * H + h) * (long)(Dv + 1) * D;
    const int rpp = MD_THREADS / lanes;                   // rows per pass
    constexpr int U = 4;                                  // passes in flight
    for (int r0 = tid / lanes; r0 - tid / lanes <= Dv; r0 += rpp * U) {
        float s[U][4], vv[U];
#pragma unroll
        for (int x = 0; x < U; ++x) {
            const int r = r0 + x * rpp;
            vv[x] = 0.f;
#pragma unroll
            for (int e = 0; e < 4; ++e) s[x][e] = 0.f;
            if (r > Dv) continue;
            vv[x] = r == Dv ? 1.f : ldf<T>(v + b * vs + (long)h * Dv + r);
            if (p <= 0) continue;                         // a sequence starts from zero
            if (vec) {
                if (li * 4 < D) {
                    const float4 t = *reinterpret_cast<const float4*>(sp + (long)r * D + li * 4);
                    s[x][0] = t.x; s[x][1] = t.y; s[x][2] = t.z; s[x][3] = t.w;
                }
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e) if (dd[e] < D) s[x][e] = sp[(long)r * D + dd[e]];
            }
        }
#pragma unroll
        for (int x = 0; x < U; ++x) {
            const int r = r0 + x * rpp;
            float acc = 0.f;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                s[x][e] = a * s[x][e] + kr[e] * vv[x];
                acc += s[x][e] * qr[e];
            }
            for (int o = lanes / 2; o > 0; o >>= 1) acc += __shfl_xor(acc, o, WAVE);
            if (r > Dv) continue;
            if (li == 0) osm[r] = acc;
            if (vec) {
                if (li * 4 < D)
                    *reinterpret_cast<float4*>(sp + (long)r * D + li * 4) =
                        make_float4(s[x][0], s[x][1], s[x][2], s[x][3]);
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e) if (dd[e] < D) sp[(long)r * D + dd[e]] = s[x][e];
            }
        }
    }
    __syncthreads();
    if (tid == 0) mstate[(long)slot * H + h] = m;         // all have read it
    const float inv = 1.f / (fmaxf(fabsf(osm[Dv]), expf(-m)) + 1e-6f);
    float ss = 0.f;
    for (int c = tid; c < Dv; c += MD_THREADS) { const float x = osm[c] * inv; ss += x * x; }
    ss = wave_sum(ss);
    if ((tid & (WAVE - 1)) == 0) red[tid / WAVE] = ss;
    __syncthreads();
    float tot = 0.f;
#pragma unroll
    for (int x = 0; x < MD_THREADS / WAVE; ++x) tot += red[x];
    const float nrm = inv / sqrtf(tot / Dv + eps);
    const T* gp = gate + b * gs + (long)h * Dv;
    for (int c = tid; c < Dv; c += MD_THREADS)
        stf<T>(op + c, osm[c] * nrm * nw[h * Dv + c] * sigmoidf_(ldf<T>(gp + c)));
}

// Long bf16 rows in chunks of GC_N tokens on the matrix cores. G_t is the running sum
// of log a inside a chunk; all exponents are differences G_t - G_s (s <= t) and never
// positive.
//   mlstm_chunk_state_kernel  E = sum_s w_s exp(G_end - G_s) k_s v_s^T (and the n row),
//                             the factor folded into the keys, three bf16 terms
//   gla_chunk_link_kernel     start states S_c (two bf16 terms), the carried state
//   mlstm_chunk_out_kernel    A_ts = (q_t k_s) w_s exp(G_t - G_s), o_t = exp(G_t) q_t S_c
//                             + sum_s A_ts v_s; n_t q_t from S_c's last row and the sums
//                             of A's rows; division, norm, weight, sigmoid gate
// Decays are one number per token and head, so they multiply the scores and the
// accumulators in fp32 and the products take q, k and v as they are.

// exclusive use of one wave: running sum of log a over the chunk's tokens (lane = token;
// tokens past the last add nothing)
DEV float chunk_decay_sum_(const float* __restrict__ ld, long tok0, int H, int h, int cnt,
                           int lane) {
    float g = lane < cnt ? ld[(tok0 + lane) * H + h] : 0.f;
#pragma unroll
    for (int o = 1; o < WAVE; o <<= 1) {
        const float x = __shfl_up(g, o, WAVE);
        if (lane >= o) g += x;
    }
    return g;
}

template <int DP, int NT>
__global__ void __launch_bounds__(256)
mlstm_chunk_state_kernel(const bf16* __restrict__ k, long ks, const bf16* __restrict__ v, long vs,
                         const float* __restrict__ ld, const float* __restrict__ wt,
                         float k_scale, const int* __restrict__ seq,
                         const int* __restrict__ nvalid, float* __restrict__ ws,
                         float* __restrict__ wdec, int S, int H, int D, int Dv, int nc) {
    __shared__ __attribute__((aligned(16))) uint16_t kt[3][DP * GC_VS];
    __shared__ __attribute__((aligned(16))) uint16_t vt[NT * 16 * GC_VS];
    __shared__ float cf[GC_N];                            // w_s exp(G_end - G_s) k_scale
    __shared__ float tot[4][DP];
    const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
    const int lr = lane & 15, lg = lane >> 4;
    const int c = blockIdx.x % nc, d0 = blockIdx.x / nc * DP, h = blockIdx.y, b = blockIdx.z;
    const int n = seq[b] < 0 ? 0 : nvalid[b];
    const int cnt = min(GC_N, n - c * GC_N);
    if (cnt <= 0) return;                                 // uniform
    const long tok0 = (long)b * S + c * GC_N;
    const int Dn = min(DP, D - d0);                       // this workgroup's key channels
    const bf16* kp = k + (long)h * D + d0;
    static_assert(4 * DP <= 256, "one (channel, 16 tokens) task per thread");
    uint4 vr[NT / 2];
    gc_load_rows_<NT * 2>(v + tok0 * vs + (long)h * Dv, vs, cnt, Dv, vr, tid);
    const int d = tid % DP, sb = tid / DP;
    float kv[16];
    if (sb < 4) {
        const int dc = min(d, Dn - 1);
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            const int m = sb * 16 + i;
            const float kk = ldf<bf16>(kp + (tok0 + min(m, cnt - 1)) * ks + dc);
            kv[i] = m < cnt && d < Dn ? kk : 0.f;
        }
    }
    if (wv == 0) {
        const float g = chunk_decay_sum_(ld, tok0, H, h, cnt, lane);
        const float end = __shfl(g, WAVE - 1, WAVE);
        cf[lane] = lane < cnt ? wt[(tok0 + lane) * H + h] * k_scale * expf(end - g) : 0.f;
        if (lane == 0 && d0 == 0) wdec[((long)b * nc + c) * H + h] = expf(end);
    }
    gc_store_vt_<NT * 2>(vr, vt, tid);
    __syncthreads();
    if (sb < 4) {
        float ns = 0.f;
        bf16x8_t t0[2], t1[2], t2[2];                     // the three terms of 16 tokens
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            const float x = kv[i] * cf[sb * 16 + i];
            ns += x;
            const __bf16 a0 = (__bf16)x;
            const float r1 = x - (float)a0;
            const __bf16 a1 = (__bf16)r1;
            t0[i >> 3][i & 7] = a0;
            t1[i >> 3][i & 7] = a1;
            t2[i >> 3][i & 7] = (__bf16)(r1 - (float)a1);
        }
        tot[sb][d] = ns;
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            const int at = d * GC_VS + sb * 16 + u * 8;
            *reinterpret_cast<bf16x8_t*>(kt[0] + at) = t0[u];
            *reinterpret_cast<bf16x8_t*>(kt[1] + at) = t1[u];
            *reinterpret_cast<bf16x8_t*>(kt[2] + at) = t2[u];
        }
    }
    __syncthreads();
    float* wp = ws + (((long)b * nc + c) * H + h) * (long)(Dv + 1) * D + d0;
    if (tid < Dn) wp[(long)Dv * D + tid] = tot[0][tid] + tot[1][tid] + tot[2][tid] + tot[3][tid];
    constexpr int DT = DP / 16;
    for (int tile = wv; tile < DT * NT; tile += 4) {
        const int dt = tile % DT, nt = tile / DT;
        if (nt * 16 >= Dv || dt * 16 >= Dn) continue;
        f32x4_t acc = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kk = 0; kk < 2; ++kk) {
            const bf16x8_t va = *reinterpret_cast<const bf16x8_t*>(
                vt + (nt * 16 + lr) * GC_VS + kk * 32 + lg * 8);
#pragma unroll
            for (int e = 2; e >= 0; --e) {                // small terms first
                const bf16x8_t kb = *reinterpret_cast<const bf16x8_t*>(
                    kt[e] + (dt * 16 + lr) * GC_VS + kk * 32 + lg * 8);
                acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(va, kb, acc, 0, 0, 0);
            }
        }
        const int dd = dt * 16 + lr;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int nn = nt * 16 + lg * 4 + r;
            if (nn < Dv && dd < Dn) wp[(long)nn * D + dd] = acc[r];
        }
    }
}

// two words of packed (high | low) bf16 terms each -> a vector of high and one of low terms
DEV void unpack_terms_(const uint4 s0, const uint4 s1, bf16x8_t& hi, bf16x8_t& lo) {
    const uint4 hv = make_uint4(
        (s0.x >> 16) | (s0.y & 0xffff0000u), (s0.z >> 16) | (s0.w & 0xffff0000u),
        (s1.x >> 16) | (s1.y & 0xffff0000u), (s1.z >> 16) | (s1.w & 0xffff0000u));
    const uint4 lv = make_uint4(
        (s0.x & 0xffffu) | (s0.y << 16), (s0.z & 0xffffu) | (s0.w << 16),
        (s1.x & 0xffffu) | (s1.y << 16), (s1.z & 0xffffu) | (s1.w << 16));
    hi = __builtin_bit_cast(bf16x8_t, hv);
    lo = __builtin_bit_cast(bf16x8_t, lv);
}

// Workgroup = (chunk, head). Wave w makes the scores of tokens 16 w .. and leaves them
// in LDS (two bf16 terms); then it owns value tiles w * NT/4 .. for all 64 tokens, so a
// start state's rows are read by one wave only.
template <int DP, int NT>
__global__ void __launch_bounds__(256, 2)
mlstm_chunk_out_kernel(const bf16* __restrict__ q, long qs, const bf16* __restrict__ k, long ks,
                       const bf16* __restrict__ v, long vs, const float* __restrict__ ld,
                       const float* __restrict__ wt, const float* __restrict__ mx, float k_scale,
                       const bf16* __restrict__ gate, long gs, const float* __restrict__ nw,
                       float eps, const int* __restrict__ seq, const int* __restrict__ nvalid,
                       const float* __restrict__ ws, bf16* __restrict__ out, int S, int H, int D,
                       int Dv, int nc) {
    constexpr int KS = DP + 8, KK = DP / 32, NTW = NT / 4, OS = NT * 16 + 4;
    constexpr int QK = 2 * GC_N * KS * 2 > GC_N * OS * 4 ? 2 * GC_N * KS * 2 : GC_N * OS * 4;
    extern __shared__ __attribute__((aligned(16))) char smc[];
    uint16_t* ql = reinterpret_cast<uint16_t*>(smc);      // GC_N * KS, then kl: the same
    uint16_t* kl = ql + GC_N * KS;
    float* ol = reinterpret_cast<float*>(smc);            // GC_N * OS, over q and k in the end
    uint16_t* vt = reinterpret_cast<uint16_t*>(smc + QK); // NT * 16 * GC_VS
    uint16_t* ah = vt + NT * 16 * GC_VS;                  // GC_N * GC_VS, rows = queries
    uint16_t* al = ah + GC_N * GC_VS;
    float* gl = reinterpret_cast<float*>(al + GC_N * GC_VS);   // G_t in base 2
    float* wl = gl + GC_N;                                // w_s k_scale
    float* iv = wl + GC_N;                                // 1 / normalizer
    float (*part)[GC_N] = reinterpret_cast<float (*)[GC_N]>(iv + GC_N);   // 4 x GC_N
    const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
    const int lr = lane & 15, lg = lane >> 4;
    const int c = blockIdx.x, h = blockIdx.y, b = blockIdx.z;
    const int n = seq[b] < 0 ? 0 : nvalid[b];
    const int cnt = min(GC_N, n - c * GC_N);
    if (cnt <= 0) return;                                 // uniform
    const long tok0 = (long)b * S + c * GC_N;
    uint4 qr[DP / 32], kr[DP / 32], vr[NT / 2];
    gc_load_rows_<DP / 8>(q + tok0 * qs + (long)h * D, qs, cnt, D, qr, tid);
    gc_load_rows_<DP / 8>(k + tok0 * ks + (long)h * D, ks, cnt, D, kr, tid);
    gc_load_rows_<NT * 2>(v + tok0 * vs + (long)h * Dv, vs, cnt, Dv, vr, tid);
    // the start state: this wave's value rows, and this lane's share of the n row
    const float* sp = ws + (((long)b * nc + c) * H + h) * (long)(Dv + 1) * D;
    uint4 sr[NTW][KK][2], nr[KK][2];
#pragma unroll
    for (int kk = 0; kk < KK; ++kk) {
        const int d = kk * 32 + lg * 8;
#pragma unroll
        for (int i = 0; i < NTW; ++i) {
            const int row = (w * NTW + i) * 16 + lr;
            sr[i][kk][0] = sr[i][kk][1] = make_uint4(0, 0, 0, 0);
            if (row < Dv && d < D) {
                const float* rp = sp + (long)row * D + d;
                sr[i][kk][0] = *reinterpret_cast<const uint4*>(rp);
                sr[i][kk][1] = *reinterpret_cast<const uint4*>(rp + 4);
            }
        }
        nr[kk][0] = nr[kk][1] = make_uint4(0, 0, 0, 0);
        if (d < D) {
            const float* rp = sp + (long)Dv * D + d;
            nr[kk][0] = *reinterpret_cast<const uint4*>(rp);
            nr[kk][1] = *reinterpret_cast<const uint4*>(rp + 4);
        }
    }
    if (w == 0) {
        gl[lane] = chunk_decay_sum_(ld, tok0, H, h, cnt, lane) * 1.4426950408889634f;
        wl[lane] = lane < cnt ? wt[(tok0 + lane) * H + h] * k_scale : 0.f;
    }
#pragma unroll
    for (int i = 0; i < DP / 32; ++i) {
        const int x = tid + i * 256;
        const int at = (x % GC_N) * KS + (x / GC_N) * 8;
        *reinterpret_cast<uint4*>(ql + at) = qr[i];
        *reinterpret_cast<uint4*>(kl + at) = kr[i];
    }
    gc_store_vt_<NT * 2>(vr, vt, tid);
    __syncthreads();
    // ---- scores of tokens 16 w + lr (a lane: keys j*16 + lg*4 .. +3)
    {
        const int t = w * 16 + lr;
        const float gt = gl[t];
        bf16x8_t qf[KK];
        float nq = 0.f;
#pragma unroll
        for (int kk = 0; kk < KK; ++kk) {
            qf[kk] = *reinterpret_cast<const bf16x8_t*>(ql + t * KS + kk * 32 + lg * 8);
            bf16x8_t hi, lo;
            unpack_terms_(nr[kk][0], nr[kk][1], hi, lo);
#pragma unroll
            for (int e = 0; e < 8; ++e) nq += (float)qf[kk][e] * ((float)hi[e] + (float)lo[e]);
        }
        nq *= exp2_(gt);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            if (j > (w | 1)) continue;                    // blocks no product reads
            f32x4_t acc = f32x4_t{0.f, 0.f, 0.f, 0.f};
            if (j <= w)
#pragma unroll
                for (int kk = 0; kk < KK; ++kk) {
                    const bf16x8_t kf = *reinterpret_cast<const bf16x8_t*>(
                        kl + (j * 16 + lr) * KS + kk * 32 + lg * 8);
                    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[kk], acc, 0, 0, 0);
                }
            union { __bf16 x[4]; uint2 u; } ph, pl;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int s = j * 16 + lg * 4 + r;
                const float a = s <= t ? acc[r] * wl[s] * exp2_(gt - gl[s]) : 0.f;
                nq += a;
                split_bf16_(a, ph.x[r], pl.x[r]);
            }
            *reinterpret_cast<uint2*>(ah + t * GC_VS + j * 16 + lg * 4) = ph.u;
            *reinterpret_cast<uint2*>(al + t * GC_VS + j * 16 + lg * 4) = pl.u;
        }
        nq += __shfl_xor(nq, 16, WAVE);
        nq += __shfl_xor(nq, 32, WAVE);
        if (lg == 0) {
            const float m = mx[(tok0 + min(t, cnt - 1)) * H + h];
            iv[t] = 1.f / (fmaxf(fabsf(nq), expf(-m)) + 1e-6f);
        }
    }
    __syncthreads();
    // ---- o = exp(G_t) q S + A v for this wave's value tiles, divided
    f32x4_t o[4][NTW];
#pragma unroll
    for (int tb = 0; tb < 4; ++tb) {
        bf16x8_t qf[KK];
#pragma unroll
        for (int kk = 0; kk < KK; ++kk)
            qf[kk] = *reinterpret_cast<const bf16x8_t*>(ql + (tb * 16 + lr) * KS + kk * 32 + lg * 8);
        const float4 g4 = *reinterpret_cast<const float4*>(gl + tb * 16 + lg * 4);
        const float eg[4] = {exp2_(g4.x), exp2_(g4.y), exp2_(g4.z), exp2_(g4.w)};
#pragma unroll
        for (int i = 0; i < NTW; ++i) {
            f32x4_t acc = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int kk = 0; kk < KK; ++kk) {
                bf16x8_t hi, lo;
                unpack_terms_(sr[i][kk][0], sr[i][kk][1], hi, lo);
                acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf[kk], lo, acc, 0, 0, 0);
                acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf[kk], hi, acc, 0, 0, 0);
            }
#pragma unroll
            for (int r = 0; r < 4; ++r) acc[r] *= eg[r];
#pragma unroll
            for (int pr = 0; pr < 2; ++pr) {
                if (pr * 2 > tb) continue;
                const bf16x8_t vb = *reinterpret_cast<const bf16x8_t*>(
                    vt + ((w * NTW + i) * 16 + lr) * GC_VS + pr * 32 + lg * 8);
                const bf16x8_t pl = *reinterpret_cast<const bf16x8_t*>(
                    al + (tb * 16 + lr) * GC_VS + pr * 32 + lg * 8);
                const bf16x8_t ph = *reinterpret_cast<const bf16x8_t*>(
                    ah + (tb * 16 + lr) * GC_VS + pr * 32 + lg * 8);
                acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pl, vb, acc, 0, 0, 0);
                acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ph, vb, acc, 0, 0, 0);
            }
            o[tb][i] = acc;
        }
    }
#pragma unroll
    for (int tb = 0; tb < 4; ++tb)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int t = tb * 16 + lg * 4 + r;
            const float inv = iv[t];
            float ss = 0.f;
#pragma unroll
            for (int i = 0; i < NTW; ++i) { o[tb][i][r] *= inv; ss += o[tb][i][r] * o[tb][i][r]; }
            ss += __shfl_xor(ss, 1, WAVE);                // channels past Dv are zero
            ss += __shfl_xor(ss, 2, WAVE);
            ss += __shfl_xor(ss, 4, WAVE);
            ss += __shfl_xor(ss, 8, WAVE);
            if (lr == 0) part[w][t] = ss;
        }
    __syncthreads();                                      // q and k are no longer read
#pragma unroll
    for (int tb = 0; tb < 4; ++tb)
#pragma unroll
        for (int r = 0; r < 4; ++r)
#pragma unroll
            for (int i = 0; i < NTW; ++i)
                ol[(tb * 16 + lg * 4 + r) * OS + (w * NTW + i) * 16 + lr] = o[tb][i][r];
    __syncthreads();
    const int D8 = Dv / 8;
    for (int x = tid; x < cnt * D8; x += 256) {
        const int t = x / D8, ch = (x % D8) * 8;
        const float inv = 1.f / sqrtf((part[0][t] + part[1][t] + part[2][t] + part[3][t]) / Dv + eps);
        float ov[8], gv[8];
        load8<float>(ol + t * OS + ch, ov);
        load8<bf16>(gate + (tok0 + t) * gs + (long)h * Dv + ch, gv);
#pragma unroll
        for (int e = 0; e < 8; ++e) ov[e] *= inv * nw[h * Dv + ch + e] * sigmoidf_(gv[e]);
        store8<bf16>(out + (tok0 + t) * (long)(H * Dv) + (long)h * Dv + ch, ov);
    }
}

static inline int grid_for(long total, int block, int cap = 8192) {
    long g = (total + block - 1) / block;
    if (g < 1) g = 1;
    return (int)(g > cap ? cap : g);
}

extern "C" {

int nx_layer_norm(const float* x, const float* w, const float* bias, void* out, int out_bf16,
                  long rows, int C, float eps, hipStream_t st) {
    if (rows <= 0) return 0;
    dim3 grid((unsigned)rows), block(LN_THREADS);
    if (out_bf16)
        layer_norm_kernel<bf16><<<grid, block, 0, st>>>(x, w, bias, (bf16*)out, rows, C, eps);
    else layer_norm_kernel<float><<<grid, block, 0, st>>>(x, w, bias, (float*)out, rows, C, eps);
    return (int)hipGetLastError();
}

int nx_add_layer_norm(float* stream, const void* y, int y_bf16, float alpha, const float* w,
                      const float* bias, float eps, void* copy, int copy_bf16, long rows, int C,
                      hipStream_t st) {
    if (rows <= 0) return 0;
    if (C <= 0) return -1;
    dim3 grid((unsigned)rows), block(LN_THREADS);
    const bool vec = (C % 8) == 0 && C <= LN_THREADS * 8 * 4 && ((uintptr_t)stream % 16) == 0 &&
                     ((uintptr_t)y % 16) == 0 && ((uintptr_t)copy % 16) == 0 &&
                     ((uintptr_t)w % 16) == 0 && ((uintptr_t)bias % 16) == 0;
#define ALA(TY, TC) stream, (const TY*)y, alpha, w, bias, eps, (TC*)copy, C
#define ALN(TY, TC) do { \
        if (!vec) add_layer_norm_kernel<TY, TC><<<grid, block, 0, st>>>(ALA(TY, TC)); \
        else if (C <= LN_THREADS * 8) \
            add_layer_norm_vec_kernel<TY, TC, 1><<<grid, block, 0, st>>>(ALA(TY, TC)); \
        else if (C <= LN_THREADS * 16) \
            add_layer_norm_vec_kernel<TY, TC, 2><<<grid, block, 0, st>>>(ALA(TY, TC)); \
        else add_layer_norm_vec_kernel<TY, TC, 4><<<grid, block, 0, st>>>(ALA(TY, TC)); } while (0)
    if (y_bf16 && copy_bf16) ALN(bf16, bf16);
    else if (y_bf16) ALN(bf16, float);
    else if (copy_bf16) ALN(float, bf16);
    else ALN(float, float);
#undef ALN
#undef ALA
    return (int)hipGetLastError();
}

int nx_short_conv(const void* x, long xs, int x_bf16, const float* w, const float* tail,
                  const int* pos, const int* seq, const int* nvalid, void* y, int y_bf16, int B,
                  int S, int C, int taps, int act_silu, int residual, const float* bias,
                  hipStream_t st) {
    const long total = (long)B * S * C;
    if (total <= 0) return 0;
    {
        // tiled path: 8-channel groups with 16-byte accesses on every row
        const int esz = x_bf16 ? 2 : 4;
        const int tiles = (S + SC_TT - 1) / SC_TT;
        const bool ok = taps >= 2 && taps <= 4 && (C % 8) == 0 && ((xs * esz) % 16) == 0 &&
                        ((uintptr_t)x % 16) == 0 && ((uintptr_t)y % 16) == 0 &&
                        ((uintptr_t)tail % 16) == 0 && (long)B * tiles <= 65535 && S >= 8;
        if (ok) {
            dim3 gt((C / 8 + 127) / 128, (unsigned)(B * tiles)), bt(128);
#define SCT(TI, TO, TP) short_conv_tile_kernel<TI, TO, TP><<<gt, bt, 0, st>>>( \
        (const TI*)x, xs, w, tail, pos, seq, nvalid, (TO*)y, S, C, tiles, act_silu, residual, bias)
#define SCTT(TI, TO) do { if (taps == 2) SCT(TI, TO, 2); else if (taps == 3) SCT(TI, TO, 3); \
                          else SCT(TI, TO, 4); } while (0)
            if (x_bf16 && y_bf16) SCTT(bf16, bf16);
            else if (x_bf16) SCTT(bf16, float);
            else if (y_bf16) SCTT(float, bf16);
            else SCTT(float, float);
#undef SCTT
#undef SCT
            return (int)hipGetLastError();
        }
    }
    dim3 grid(grid_for(total, 256)), block(256);
#define SC(TI, TO) short_conv_kernel<TI, TO><<<grid, block, 0, st>>>( \
        (const TI*)x, xs, w, tail, pos, seq, (TO*)y, B, S, C, taps, act_silu, residual, bias)
    if (x_bf16 && y_bf16) SC(bf16, bf16);
    else if (x_bf16) SC(bf16, float);
    else if (y_bf16) SC(float, bf16);
    else SC(float, float);
#undef SC
    return (int)hipGetLastError();
}

int nx_short_conv_commit(const void* x, long xs, int x_bf16, float* tail, const int* pos,
                         const int* seq, const int* nvalid, int B, int S, int C, int R,
                         hipStream_t st) {
    const long total = (long)B * C;
    if (total <= 0 || R <= 0) return 0;
    dim3 grid((unsigned)((total + 255) / 256)), block(256);
    if (x_bf16) short_conv_commit_kernel<bf16><<<grid, block, 0, st>>>(
        (const bf16*)x, xs, tail, pos, seq, nvalid, B, S, C, R);
    else short_conv_commit_kernel<float><<<grid, block, 0, st>>>(
        (const float*)x, xs, tail, pos, seq, nvalid, B, S, C, R);
    return (int)hipGetLastError();
}

int nx_paged_kv_write(void* kc, void* vc, const void* k, long kstride, const void* v,
                      long vstride, int is_bf16, const int* slots, long N, int GDk, int GDv,
                      long nslots, hipStream_t st) {
    const long total = N * (GDk + GDv);
    if (total <= 0) return 0;
    dim3 grid(grid_for(total, 256)), block(256);
    if (is_bf16) paged_kv_write_kernel<bf16><<<grid, block, 0, st>>>(
        (bf16*)kc, (bf16*)vc, (const bf16*)k, kstride, (const bf16*)v, vstride, slots, N, GDk,
        GDv, nslots);
    else paged_kv_write_kernel<float><<<grid, block, 0, st>>>(
        (float*)kc, (float*)vc, (const float*)k, kstride, (const float*)v, vstride, slots, N,
        GDk, GDv, nslots);
    return (int)hipGetLastError();
}

int nx_paged_attn(const void* q, long qstride, const void* kc, long ktok, long khead,
                  const void* vc, long vtok, long vhead, const int* pos, const int* seq,
                  const int* btab, int max_blocks, const float* r1, const float* r2,
                  const float* sink, const void* gate, long gstride, void* out, int io_bf16,
                  int out_bf16, int B, int S, int H, int G, int Dk, int Dv, int bsz,
                  float scale, int window, int keep, float cap, float qt_coef, int qt_every,
                  float* ws, int nks, int ghead, int cmask, hipStream_t st) {
    if ((long)B * S <= 0) return 0;
    if (Dv > WAVE * 8 || H % G != 0 || Dk <= 0 || Dv <= 0) return -1;
    if (!io_bf16 && out_bf16) return -2;
    if (r2 != nullptr && r1 == nullptr) return -4;
    if (cmask < 0 || window < 1) return -7;
    const int esz = io_bf16 ? 2 : 4;
    const int vecn = 16 / esz;                            // elements per 16-byte load
    const bool k_al = (Dk % 8) == 0 && (ktok % vecn) == 0 && (khead % vecn) == 0 &&
                      ((uintptr_t)kc % 16) == 0;
    const bool v_al = (Dv % 8) == 0 && (vtok % vecn) == 0 && (vhead % vecn) == 0 &&
                      ((uintptr_t)vc % 16) == 0;
    if (io_bf16 && out_bf16 && S == 1 && G == 1 && vc == kc && vtok == ktok && k_al && v_al &&
        !r1 && (!gate || ghead) && cap <= 0.f && qt_every <= 0 && keep == 0 && H >= 8 &&
        Dk <= 640 && (qstride % 8) == 0 && ((uintptr_t)q % 16) == 0) {
        // latent caches, single-token steps: one workgroup per token reads each
        // key row once and covers 512 value channels
        const int dkp = (Dk + 31) & ~31;
        const int nsplit = (Dv + 511) / 512, hch = (H + 15) / 16;
        if (nks < 1 || !ws) nks = 1;
        if (nks > 8) return -6;
        dim3 gl(S * nks, hch * nsplit, B), bl(256);
#define LD(DKV) do { \
            const size_t lsh = (size_t)(LD_KT * (DKV + 8) + 4 * LD_VW * (LD_KT + 8)) * 2; \
            static bool attr_set = false; \
            if (!attr_set) { \
                if (hipFuncSetAttribute((const void*)latent_decode_mfma_kernel<DKV>, \
                        hipFuncAttributeMaxDynamicSharedMemorySize, (int)lsh) != hipSuccess) return -5; \
                attr_set = true; \
            } \
            latent_decode_mfma_kernel<DKV><<<gl, bl, lsh, st>>>( \
                (const bf16*)q, qstride, (const bf16*)kc, ktok, pos, seq, btab, max_blocks, sink, \
                (bf16*)out, H, Dk, Dv, bsz, S, scale, nsplit, nks, ws, window, cmask, \
                (const bf16*)gate, gstride); } while (0)
        if (dkp <= 128) LD(128);
        else if (dkp <= 256) LD(256);
        else if (dkp <= 384) LD(384);
        else if (dkp <= 576) LD(576);
        else LD(640);
#undef LD
        if (nks > 1) {
            const long waves = (long)B * S * H * ((Dv + LM_W - 1) / LM_W);
            latent_decode_merge_kernel<<<(unsigned)((waves + 3) / 4), 4 * WAVE, 0, st>>>(
                ws, sink, pos, seq, (bf16*)out, (long)B * S, S, H, Dv, nks, (const bf16*)gate,
                gstride);
        }
        return (int)hipGetLastError();
    }
    {
        // matrix-core path: bf16 steps with prompt portions (any head sizes in
        // multiples of 8: keys up to 640 wide, wide values split over
        // workgroups), and single-token steps of wide multi-query layers, whose
        // many heads per cache row fill the 16-row tiles
        const int rp = H / G;
        const bool rep_ok = rp <= MA_ROWS;       // rows beyond QT*rep stay idle
        const int dkp = (Dk + 31) & ~31, dvp = (Dv + 31) & ~31;
        const bool wide = dkp > 192 || dvp > 128;
        const bool dk_ok = dkp <= 640;
        const bool steps_ok = S > 1 || (wide && rp >= 8);
        if (io_bf16 && out_bf16 && steps_ok && rep_ok && dk_ok && k_al && v_al &&
            (qstride % 8) == 0 && ((uintptr_t)q % 16) == 0) {
            const int QTm = MA_ROWS / rp;
            const int nsplit = wide ? (Dv + 127) / 128 : 1;
            dim3 gm((S + QTm - 1) / QTm, G * nsplit, B), bm(256);
#define MA(DKV, DVV, KTV) paged_attn_mfma_kernel<DKV, DVV, KTV, (KTV == 32 || (DKV == 192 && DVV == 128))><<<gm, bm, 0, st>>>( \
        (const bf16*)q, qstride, (const bf16*)kc, (const bf16*)vc, pos, seq, btab, max_blocks, \
        r1, r2, (const bf16*)gate, gstride, (bf16*)out, H, G, Dk, Dv, bsz, S, scale, window, \
        keep, QTm, ktok, khead, vtok, vhead, sink, cap, qt_coef, qt_every, nsplit, ghead, cmask)
#define MAV(DKV) do { if (dvp == 32) MA(DKV, 32, 64); else if (dvp == 64) MA(DKV, 64, 64); \
                      else if (dvp == 96) MA(DKV, 96, 64); else MA(DKV, 128, 64); } while (0)
            if (wide) {
                if (dkp <= 128) MA(128, 128, 64);
                else if (dkp <= 192) MA(192, 128, 64);
                else if (dkp <= 256) MA(256, 128, 32);
                else if (dkp <= 384) MA(384, 128, 32);
                else if (dkp <= 576) MA(576, 128, 32);
                else MA(640, 128, 32);
            }
            else if (dkp == 32) MAV(32);
            else if (dkp == 64) MAV(64);
            else if (dkp == 96) MAV(96);
            else if (dkp == 128) MAV(128);
            else MAV(192);
#undef MAV
#undef MA
            return (int)hipGetLastError();
        }
    }
    const bool dec = S == 1;                              // pure decode step
    const int NQ = dec ? 4 : 16, NW = dec ? 16 : 4;
    const int rep = H / G;
    const int HPW = rep < NQ ? rep : NQ;                  // query heads per workgroup
    const int QT = NQ / HPW;                              // tokens per workgroup
    const int chunks = (rep + HPW - 1) / HPW;
    const int DkP = (Dk + 7) & ~7;
    dim3 grid((S + QT - 1) / QT, G * chunks, B), block(NW * WAVE);
    // decode shape: 8 value channels per lane when they tile a wave evenly
    int lpr = 0;
    if (dec && v_al) {
        const int l = Dv / 8;
        if (l <= WAVE && (l & (l - 1)) == 0) lpr = l;
    }
    int pws = (lpr > 0 && NQ * Dv > WAVE * NQ) ? NQ * Dv : WAVE * NQ;
    long ptile = (long)NW * pws;
    const long marea = (long)(NW / 2) * NQ * (Dv + 2);
    size_t sh = (size_t)(NQ * DkP + (ptile > marea ? ptile : marea)) * sizeof(float);
    if (sh > 60 * 1024 && lpr > 0) {                      // wide values: scalar P.V
        lpr = 0;
        pws = WAVE * NQ;
        ptile = (long)NW * pws;
        sh = (size_t)(NQ * DkP + (ptile > marea ? ptile : marea)) * sizeof(float);
    }
    if (sh > 150 * 1024) return -3;
    const int kvec = k_al ? 1 : 0;
    // beyond the default 64 KB of dynamic LDS a kernel has to be told its limit
#define WA(T, TO, MR, Q, W) if (sh > 60 * 1024 && hipFuncSetAttribute( \
        (const void*)window_attn_kernel<T, TO, MR, Q, W>, \
        hipFuncAttributeMaxDynamicSharedMemorySize, (int)sh) != hipSuccess) return -5; \
    window_attn_kernel<T, TO, MR, Q, W><<<grid, block, sh, st>>>( \
        (const T*)q, qstride, (const T*)kc, (const T*)vc, pos, seq, btab, max_blocks, r1, r2, \
        (const T*)gate, gstride, (TO*)out, H, G, Dk, Dv, bsz, S, scale, window, keep, HPW, QT, \
        chunks, lpr, pws, ktok, khead, vtok, vhead, kvec, sink, cap, qt_coef, qt_every, ghead, \
        cmask)
#define WAS(T, TO, MR) do { if (dec) { WA(T, TO, MR, 4, 16); } else { WA(T, TO, MR, 16, 4); } } while (0)
#define WAM(T, TO) do { if (Dv <= 2 * WAVE) WAS(T, TO, 2); else if (Dv <= 4 * WAVE) WAS(T, TO, 4); \
                        else WAS(T, TO, 8); } while (0)
    if (io_bf16 && out_bf16) WAM(bf16, bf16);
    else if (io_bf16) WAM(bf16, float);
    else WAM(float, float);
#undef WAM
#undef WAS
#undef WA
    return (int)hipGetLastError();
}

int nx_gated_delta(const float* qkv, long cstride, const void* beta, long bstride, const void* a,
                   long astride, const void* gate, long gstride, const float* dt_bias,
                   const float* a_log, const float* norm_w, float eps, float* state,
                   const int* pos, const int* seq, const int* nvalid, float* prep, long PS,
                   float* obuf, void* out, int in_bf16, int B, int S, int H, int G, int D,
                   int Dv, int per_head, int gate_silu, hipStream_t st) {
    if (B <= 0 || S <= 0) return 0;
    if (D > 256 || H % G != 0 || PS < (long)(2 * G + H) * D + H + G) return -1;
    const long ntok = (long)B * S;
    {
        const long waves = ntok * (2 * G + H);
        dim3 g0((unsigned)((waves + 3) / 4)), b0(4 * WAVE);
        if (in_bf16) delta_prep_kernel<bf16><<<g0, b0, 0, st>>>(
            qkv, cstride, (const bf16*)beta, bstride, (const bf16*)a, astride, dt_bias, a_log,
            pos, seq, prep, PS, ntok, S, H, G, D, per_head);
        else delta_prep_kernel<float><<<g0, b0, 0, st>>>(
            qkv, cstride, (const float*)beta, bstride, (const float*)a, astride, dt_bias, a_log,
            pos, seq, prep, PS, ntok, S, H, G, D, per_head);
        int rc = (int)hipGetLastError();
        if (rc) return rc;
    }
    const int parts = D <= 32 ? 8 : 16;
    const int cw = GD_THREADS / parts;
    dim3 grid((Dv + cw - 1) / cw, H, B), block(GD_THREADS);
#define GD(DKV, TCV, PV) gated_delta_kernel<DKV, TCV, PV><<<grid, block, 0, st>>>( \
        qkv, cstride, prep, PS, state, pos, seq, nvalid, obuf, S, H, G, D, Dv)
    if (D <= 32) GD(32, 16, 8);
    else if (D <= 64) GD(64, 16, 16);
    else if (D <= 128) GD(128, 16, 16);
    else GD(256, 8, 16);
#undef GD
    int rc = (int)hipGetLastError();
    if (rc) return rc;
    const long waves = ntok * H;
    dim3 g2((unsigned)((waves + 3) / 4)), b2(4 * WAVE);
    if (in_bf16) gated_rmsnorm_kernel<bf16><<<g2, b2, 0, st>>>(
        obuf, (const bf16*)gate, gstride, norm_w, eps, pos, seq, (bf16*)out, ntok, S, H, Dv,
        gate_silu);
    else gated_rmsnorm_kernel<float><<<g2, b2, 0, st>>>(
        obuf, (const float*)gate, gstride, norm_w, eps, pos, seq, (float*)out, ntok, S, H, Dv,
        gate_silu);
    return (int)hipGetLastError();
}

int nx_softcap(const void* in, int in_bf16, float* out, long n, float cap, hipStream_t st) {
    if (n <= 0) return 0;
    dim3 grid(grid_for(n, 256)), block(256);
    if (in_bf16) softcap_kernel<bf16><<<grid, block, 0, st>>>((const bf16*)in, out, n, cap);
    else softcap_kernel<float><<<grid, block, 0, st>>>((const float*)in, out, n, cap);
    return (int)hipGetLastError();
}

int nx_residual_add(float* x, const void* a, float sa, const void* b, float sb, int is_bf16,
                    long n, hipStream_t st) {
    if (n <= 0) return 0;
    dim3 grid(grid_for(n, 256)), block(256);
    if (is_bf16) residual_add_kernel<bf16><<<grid, block, 0, st>>>(
        x, (const bf16*)a, sa, (const bf16*)b, sb, n);
    else residual_add_kernel<float><<<grid, block, 0, st>>>(
        x, (const float*)a, sa, (const float*)b, sb, n);
    return (int)hipGetLastError();
}

int nx_gelu_mul(const void* gu, void* out, int is_bf16, long rows, int I, int silu,
                hipStream_t st) {
    if (rows <= 0) return 0;
    const bool vec = (I % 8) == 0 && ((uintptr_t)gu % 16) == 0 && ((uintptr_t)out % 16) == 0;
    dim3 gv((I / 8 + 255) / 256, (unsigned)(rows > 32768 ? 32768 : rows));
    dim3 grid(grid_for(rows * I, 256)), block(256);
#define GM(T, A) do { if (vec) gelu_mul_vec_kernel<T, A><<<gv, block, 0, st>>>( \
        (const T*)gu, (T*)out, rows, I); \
    else gelu_mul_kernel<T, A><<<grid, block, 0, st>>>((const T*)gu, (T*)out, rows, I); } while (0)
    if (is_bf16) { if (silu) GM(bf16, 1); else GM(bf16, 0); }
    else { if (silu) GM(float, 1); else GM(float, 0); }
#undef GM
    return (int)hipGetLastError();
}

int nx_rms_norm(const void* x, long xs, int x_bf16, const float* w, int one_plus, float eps,
                void* out, long os, int out_bf16, long rows, int C, hipStream_t st) {
    if (rows <= 0) return 0;
    dim3 grid((unsigned)rows), block(LN_THREADS);
    const int xe = x_bf16 ? 2 : 4, oe = out_bf16 ? 2 : 4;
    const bool vec = (C % 8) == 0 && ((uintptr_t)x % 16) == 0 && ((uintptr_t)out % 16) == 0 &&
                     ((xs * xe) % 16) == 0 && ((os * oe) % 16) == 0 && ((uintptr_t)w % 16) == 0;
#define RN(TI, TO) do { if (vec) rms_norm_vec_kernel<TI, TO><<<grid, block, 0, st>>>( \
        (const TI*)x, xs, w, one_plus, eps, (TO*)out, os, C); \
    else rms_norm_kernel<TI, TO><<<grid, block, 0, st>>>( \
        (const TI*)x, xs, w, one_plus, eps, (TO*)out, os, C); } while (0)
    if (x_bf16 && out_bf16) RN(bf16, bf16);
    else if (x_bf16) RN(bf16, float);
    else if (out_bf16) RN(float, bf16);
    else RN(float, float);
#undef RN
    return (int)hipGetLastError();
}

int nx_add_rms_norm(float* stream, const void* y, int y_bf16, const float* w, int one_plus,
                    float eps, void* copy, int copy_bf16, const void* extra, const float* coef,
                    long cs, int nc, const float* next_w, long rows, int C, hipStream_t st) {
    if (rows <= 0) return 0;
    if ((extra == nullptr) != (coef == nullptr)) return -1;
    dim3 grid((unsigned)rows), block(LN_THREADS);
    const bool vec = (C % 8) == 0 && ((uintptr_t)stream % 16) == 0 && ((uintptr_t)y % 16) == 0 &&
                     ((uintptr_t)copy % 16) == 0 && ((uintptr_t)w % 16) == 0 &&
                     ((uintptr_t)extra % 16) == 0 && ((uintptr_t)next_w % 16) == 0;
#define ARN(K, TY, TC) K<TY, TC><<<grid, block, 0, st>>>(stream, (const TY*)y, w, one_plus, eps, \
        (TC*)copy, (const TY*)extra, coef, cs, nc, next_w, C)
#define ARN2(K) do { if (y_bf16 && copy_bf16) ARN(K, bf16, bf16); else if (y_bf16) ARN(K, bf16, float); \
                     else if (copy_bf16) ARN(K, float, bf16); else ARN(K, float, float); } while (0)
    if (vec) ARN2(add_rms_norm_vec_kernel);
    else ARN2(add_rms_norm_kernel);
#undef ARN2
#undef ARN
    return (int)hipGetLastError();
}

int nx_rope_pairs(const void* x, long xt, long xh, int x_bf16, void* out, long ot, long oh,
                  int out_bf16, const int* pos, const float* inv_freq, int half, int split,
                  long ntok, int N, int C, hipStream_t st) {
    const long total = ntok * N * (C - half);
    if (total <= 0) return 0;
    if (2 * half > C) return -1;
    dim3 grid(grid_for(total, 256)), block(256);
#define RP(TI, TO) rope_pairs_kernel<TI, TO><<<grid, block, 0, st>>>( \
        (const TI*)x, xt, xh, (TO*)out, ot, oh, pos, inv_freq, half, split, ntok, N, C)
    if (x_bf16 && out_bf16) RP(bf16, bf16);
    else if (x_bf16) RP(bf16, float);
    else if (out_bf16) RP(float, bf16);
    else RP(float, float);
#undef RP
    return (int)hipGetLastError();
}

int nx_clamped_glu(const void* gu, void* out, int is_bf16, long rows, int I, float limit,
                   float alpha, hipStream_t st) {
    if (rows <= 0) return 0;
    if ((I % 8) == 0 && ((uintptr_t)gu % 16) == 0 && ((uintptr_t)out % 16) == 0) {
        dim3 gv((I / 8 + 255) / 256, (unsigned)(rows > 32768 ? 32768 : rows)), bv(256);
        if (is_bf16) clamped_glu_vec_kernel<bf16><<<gv, bv, 0, st>>>(
            (const bf16*)gu, (bf16*)out, rows, I, limit, alpha);
        else clamped_glu_vec_kernel<float><<<gv, bv, 0, st>>>(
            (const float*)gu, (float*)out, rows, I, limit, alpha);
        return (int)hipGetLastError();
    }
    dim3 grid(grid_for(rows * I, 256)), block(256);
    if (is_bf16) clamped_glu_kernel<bf16><<<grid, block, 0, st>>>(
        (const bf16*)gu, (bf16*)out, rows, I, limit, alpha);
    else clamped_glu_kernel<float><<<grid, block, 0, st>>>(
        (const float*)gu, (float*)out, rows, I, limit, alpha);
    return (int)hipGetLastError();
}

int nx_head_norm_rope(const void* x, long xt, long xh, int x_bf16, void* out, int out_bf16,
                      const int* pos, const float* nw, float eps, const float* inv_freq,
                      int half, float mscale, long ntok, int N, int C, hipStream_t st) {
    if (ntok * N <= 0) return 0;
    if (C > HN_MAXC || 2 * half > C || (half > 0 && !inv_freq)) return -1;
    const long waves = ntok * N;
    dim3 grid((unsigned)((waves + HN_WAVES - 1) / HN_WAVES)), block(HN_WAVES * WAVE);
#define HN(TI, TO) head_norm_rope_kernel<TI, TO><<<grid, block, 0, st>>>( \
        (const TI*)x, xt, xh, (TO*)out, pos, nw, eps, inv_freq, half, mscale, ntok, N, C)
    if (x_bf16 && out_bf16) HN(bf16, bf16);
    else if (x_bf16) HN(bf16, float);
    else if (out_bf16) HN(float, bf16);
    else HN(float, float);
#undef HN
    return (int)hipGetLastError();
}

int nx_decay_scan(const void* q, long qs, const void* k, long ks, const void* v, long vs,
                  int in_bf16, const void* dt, long dts, int dt_bf16, const float* dt_bias,
                  const float* a_log, const float* head_decay, float k_scale, const float* skip,
                  float* state, const int* pos, const int* seq, const int* nvalid, float* out,
                  int B, int S, int H, int G, int D, int Dv, float* ws, float* wdec, int nseg,
                  int seglen, int kind, const float* wgt, hipStream_t st) {
    if ((long)B * S <= 0) return 0;
    if (D <= 0 || Dv <= 0 || G <= 0 || H % G != 0 || D > 256) return -1;
    if ((dt == nullptr) == (head_decay == nullptr)) return -2;
    if (dt && kind == 0 && (!dt_bias || !a_log)) return -2;
    if (kind != 0 && (!dt || dt_bf16 || a_log || skip)) return -2;
    if (kind < 0 || kind > 2 || (kind == 2 && (!wgt || Dv < 2))) return -2;
    if (H > 65535 || B > 65535) return -3;
    // the kernel reads state rows 16 bytes at a time when dim % 4 == 0
    if (((uintptr_t)state % 16) != 0 || ((uintptr_t)ws % 16) != 0) return -5;
    if (nseg < 1 || (nseg > 1 && (!ws || !wdec || seglen <= 0 || (long)nseg * seglen < S)))
        return -4;
    const int cb = (Dv + 15) / 16;
    dim3 grid(cb * nseg, H, B), block(256);
#define DSK(T, TD, RV, MD, CHV) decay_scan_kernel<T, TD, RV, MD, CHV><<<grid, block, 0, st>>>( \
        (const T*)q, qs, (const T*)k, ks, (const T*)v, vs, (const TD*)dt, dts, dt_bias, a_log, \
        head_decay, k_scale, skip, state, pos, seq, nvalid, out, S, H, G, D, Dv, ws, wdec, nseg, \
        seglen, wgt)
#define DSR(T, TD, MD, CHV) do { if (D <= 16) DSK(T, TD, 1, MD, CHV); \
        else if (D <= 32) DSK(T, TD, 2, MD, CHV); \
        else if (D <= 64) DSK(T, TD, 4, MD, CHV); else if (D <= 128) DSK(T, TD, 8, MD, CHV); \
        else DSK(T, TD, 16, MD, CHV); } while (0)
#define DST(MD) do { \
        if (in_bf16) { if (dt_bf16) DSR(bf16, bf16, MD, 0); else DSR(bf16, float, MD, 0); } \
        else { if (dt_bf16) DSR(float, bf16, MD, 0); else DSR(float, float, MD, 0); } } while (0)
#define DSC(MD) do { if (kind == 0) DST(MD); \
        else if (kind == 1) { if (in_bf16) DSR(bf16, float, MD, 1); else DSR(float, float, MD, 1); } \
        else { if (in_bf16) DSR(bf16, float, MD, 2); else DSR(float, float, MD, 2); } } while (0)
    if (nseg == 1) {
        DSC(0);
    } else {
        DSC(1);
        const long per_head = (long)Dv * D;
        decay_scan_link_kernel<<<grid_for((long)B * H * per_head, 256), 256, 0, st>>>(
            ws, wdec, state, pos, seq, nvalid, B, S, H, per_head, nseg, kind == 1 ? D : 1);
        DSC(2);
    }
#undef DSC
#undef DST
#undef DSR
#undef DSK
    return (int)hipGetLastError();
}

int nx_low_rank_decay(const void* low, long ls, const void* w, int is_bf16, const float* bias,
                      float inv_tau, float* out, long rows, int C, int rank, hipStream_t st) {
    if (rows * C <= 0) return 0;
    if (!bias || rank <= 0) return -1;
    const int vec = (rank % 8) == 0 && ((uintptr_t)w % 16) == 0;
    const int tt = rows <= 512 ? 2 : 16;
    const long gy = (rows + tt - 1) / tt;
    dim3 grid((C + 255) / 256, (unsigned)(gy > 32768 ? 32768 : gy)), block(256);
#define LRD(T, TT) low_rank_decay_kernel<T, TT><<<grid, block, 0, st>>>( \
        (const T*)low, ls, (const T*)w, vec, bias, inv_tau, out, rows, C, rank)
    if (is_bf16) { if (tt == 2) LRD(bf16, 2); else LRD(bf16, 16); }
    else { if (tt == 2) LRD(float, 2); else LRD(float, 16); }
#undef LRD
    return (int)hipGetLastError();
}

// chunked form of the channel-decay recurrence with the gated read-out norm fused:
// bf16 q/k/v/gate/out, D and Dv multiples of 8 up to 128
int nx_gla_chunked(const void* q, long qs, const void* k, long ks, const void* v, long vs,
                   const float* ld, float k_scale, const void* gate, long gs, const float* nw,
                   float eps, float* state, const int* pos, const int* seq, const int* nvalid,
                   float* ws, float* wdec, void* out, int B, int S, int H, int D, int Dv,
                   hipStream_t st) {
    if ((long)B * S <= 0) return 0;
    if (D <= 0 || Dv <= 0 || D > 128 || Dv > 128 || (D % 8) || (Dv % 8)) return -1;
    if ((qs % 8) || (ks % 8) || (vs % 8) || ((uintptr_t)q % 16) || ((uintptr_t)k % 16) ||
        ((uintptr_t)v % 16) || ((uintptr_t)ws % 16) || !gate || !nw) return -2;
    const int nc = (S + GC_N - 1) / GC_N;
    if (H > 65535 || B > 65535) return -3;
    dim3 grid(nc, H, B), block(256);
#define GC(DPV, NT) do { \
        constexpr int DPB = DPV < 64 ? DPV : 64; \
        const size_t lsh = (size_t)(GC_N * (DPV + 4) + 4 * DPV) * 4 + \
                           (size_t)(GC_N * (DPV + 8) + NT * 16 * GC_VS) * 2; \
        static bool attr_set = false; \
        if (!attr_set) { \
            if (hipFuncSetAttribute((const void*)gla_chunk_out_kernel<DPV, NT>, \
                    hipFuncAttributeMaxDynamicSharedMemorySize, (int)lsh) != hipSuccess) return -5; \
            attr_set = true; \
        } \
        dim3 gst(nc * ((D + DPB - 1) / DPB), H, B); \
        gla_chunk_state_kernel<DPB, NT><<<gst, block, 0, st>>>( \
            (const bf16*)k, ks, (const bf16*)v, vs, ld, k_scale, pos, seq, nvalid, ws, wdec, S, H, \
            D, Dv, nc); \
        gla_chunk_link_kernel<<<grid_for((long)B * H * Dv * D, 256), 256, 0, st>>>( \
            ws, wdec, state, pos, seq, nvalid, B, S, H, D, (long)Dv * D, nc); \
        gla_chunk_out_kernel<DPV, NT><<<grid, block, lsh, st>>>( \
            (const bf16*)q, qs, (const bf16*)k, ks, (const bf16*)v, vs, ld, k_scale, \
            (const bf16*)gate, gs, nw, eps, seq, nvalid, ws, (bf16*)out, S, H, D, Dv, nc); } while (0)
#define GCN(DPV) do { if (Dv <= 64) GC(DPV, 4); else GC(DPV, 8); } while (0)
    if (D <= 32) GCN(32); else if (D <= 64) GCN(64); else GCN(128);
#undef GCN
#undef GC
    return (int)hipGetLastError();
}

int nx_group_gated_norm(const float* y, const void* gate, long gs, int gate_bf16, const float* w,
                        float eps, int groups, int gate_first, int wshared, void* out,
                        int out_bf16, long rows, int C, hipStream_t st) {
    if (rows <= 0) return 0;
    if (groups <= 0 || C % groups != 0) return -1;
    const long waves = rows * groups;
    dim3 grid((unsigned)((waves + 3) / 4)), block(4 * WAVE);
#define GN(TG, TO) group_gated_norm_kernel<TG, TO><<<grid, block, 0, st>>>( \
        y, (const TG*)gate, gs, w, eps, groups, gate_first, wshared, (TO*)out, rows, C)
    if (gate_bf16 && out_bf16) GN(bf16, bf16);
    else if (gate_bf16) GN(bf16, float);
    else if (out_bf16) GN(float, bf16);
    else GN(float, float);
#undef GN
    return (int)hipGetLastError();
}

int nx_group_router(const float* logits, long ls, int E, int extra, int top, int ngroups,
                    int keep, float scale, int normalize, const float* corr, int sig, int gtwo,
                    float norm_eps, float* dense, int* idx, float* wts, long T, hipStream_t st) {
    if (T <= 0) return 0;
    if (E <= 0 || top <= 0 || top > E || top > WAVE || ngroups <= 0 || E % ngroups != 0 ||
        keep <= 0 || keep > ngroups || (long)top > (long)(E / ngroups) * keep) return -1;
    const size_t sh = (size_t)RT_WAVES * (2 * E + ngroups) * sizeof(float);
    if (sh > 60 * 1024) return -2;
    dim3 grid((unsigned)((T + RT_WAVES - 1) / RT_WAVES)), block(RT_WAVES * WAVE);
    group_router_kernel<<<grid, block, sh, st>>>(logits, ls, E, extra, top, ngroups, keep, scale,
                                                 normalize, corr, sig, gtwo, norm_eps, dense, idx,
                                                 wts, T);
    return (int)hipGetLastError();
}

int nx_router_fused(const void* x, long xs, int x_bf16, const float* w, int W, int E, int extra,
                    int top, int ngroups, int keep, float scale, int normalize, const float* corr,
                    const float* bias, int sig, int gtwo, float norm_eps, float* dense, int* idx,
                    float* wts, long T, hipStream_t st) {
    if (T <= 0) return 0;
    if (E <= 0 || top <= 0 || top > E || top > WAVE || ngroups <= 0 || E % ngroups != 0 ||
        keep <= 0 || keep > ngroups || (long)top > (long)(E / ngroups) * keep || W <= 0) return -1;
    const size_t sh = (size_t)(3 * E + extra + ngroups) * sizeof(float);
    if (sh > 60 * 1024) return -2;
    const int vecn = x_bf16 ? 8 : 4;
    const int vec = (W % 8) == 0 && (xs % vecn) == 0 && ((uintptr_t)x % 16) == 0 &&
                    ((uintptr_t)w % 16) == 0;
    dim3 grid((unsigned)T), block(RT_WAVES * WAVE);
    if (x_bf16) router_fused_kernel<bf16><<<grid, block, sh, st>>>(
        (const bf16*)x, xs, w, W, vec, E, extra, top, ngroups, keep, scale, normalize, corr, bias,
        sig, gtwo, norm_eps, dense, idx, wts);
    else router_fused_kernel<float><<<grid, block, sh, st>>>(
        (const float*)x, xs, w, W, vec, E, extra, top, ngroups, keep, scale, normalize, corr, bias,
        sig, gtwo, norm_eps, dense, idx, wts);
    return (int)hipGetLastError();
}

int nx_latent_row(const void* x, long xs, int is_bf16, const float* w, float eps,
                  const float* inv_freq, int half, int split, const int* pos, const int* slots,
                  void* cache, long nslots, void* row, long rs, long ntok, int C, int R, hipStream_t st) {
    if (ntok <= 0) return 0;
    if (C <= 0 || R < 0 || 2 * half > R || (half > 0 && !inv_freq)) return -1;
    dim3 grid((unsigned)((ntok + 3) / 4)), block(4 * WAVE);
    if (is_bf16) latent_row_kernel<bf16><<<grid, block, 0, st>>>(
        (const bf16*)x, xs, w, eps, inv_freq, half, split, pos, slots, (bf16*)cache, nslots, (bf16*)row,
        rs, ntok, C, R);
    else latent_row_kernel<float><<<grid, block, 0, st>>>(
        (const float*)x, xs, w, eps, inv_freq, half, split, pos, slots, (float*)cache, nslots,
        (float*)row, rs, ntok, C, R);
    return (int)hipGetLastError();
}

int nx_act_scale(const void* x, int is_bf16, const float* gates, int gcols, int ff, int E,
                 int act, void* out, long rows, int C, hipStream_t st) {
    if (rows * C <= 0) return 0;
    if (ff <= 0 || (gates && gcols < E) || act < 0 || act > 1) return -1;
    const bool vec = (C % 8) == 0 && (ff % 8) == 0 && ((uintptr_t)x % 16) == 0 &&
                     ((uintptr_t)out % 16) == 0;
    dim3 grid(grid_for(vec ? rows * (C / 8) : rows * C, 256)), block(256);
#define AS(T, A) do { if (vec) act_scale_vec_kernel<T, A><<<grid, block, 0, st>>>( \
        (const T*)x, gates, gcols, ff, E, (T*)out, rows, C); \
    else act_scale_kernel<T, A><<<grid, block, 0, st>>>( \
        (const T*)x, gates, gcols, ff, E, (T*)out, rows, C); } while (0)
    if (is_bf16) { if (act) AS(bf16, 1); else AS(bf16, 0); }
    else { if (act) AS(float, 1); else AS(float, 0); }
#undef AS
    return (int)hipGetLastError();
}

int nx_glu_scale(const void* x, int is_bf16, const float* gates, long gs, int ff, int E, int act,
                 float limit, float slimit, float alpha, void* out, long rows, int C,
                 hipStream_t st) {
    if (rows * C <= 0) return 0;
    if (E < 0 || (E > 0 && (ff <= 0 || !gates)) || (long)E * ff > C || act < 0 || act > 1) return -1;
    if (E == 0) ff = 8;
    const bool vec = (C % 8) == 0 && (ff % 8) == 0 && ((uintptr_t)x % 16) == 0 &&
                     ((uintptr_t)out % 16) == 0;
    dim3 grid(grid_for(vec ? rows * (C / 8) : rows * C, 256)), block(256);
#define GS(T, A) do { if (vec) glu_scale_vec_kernel<T, A><<<grid, block, 0, st>>>( \
        (const T*)x, gates, gs, ff, E, limit, slimit, alpha, (T*)out, rows, C); \
    else glu_scale_kernel<T, A><<<grid, block, 0, st>>>( \
        (const T*)x, gates, gs, ff, E, limit, slimit, alpha, (T*)out, rows, C); } while (0)
    if (is_bf16) { if (act) GS(bf16, 1); else GS(bf16, 0); }
    else { if (act) GS(float, 1); else GS(float, 0); }
#undef GS
    return (int)hipGetLastError();
}

int nx_sigmoid_gate(void* y, const void* gate, long gs, int is_bf16, long rows, int C,
                    hipStream_t st) {
    if (rows * C <= 0) return 0;
    const int vecn = is_bf16 ? 8 : 4;                     // elements per 16 bytes
    const int vec = (C % 8) == 0 && (gs % vecn) == 0 && ((uintptr_t)y % 16) == 0 &&
                    ((uintptr_t)gate % 16) == 0;
    dim3 grid(grid_for(vec ? rows * (C / 8) : rows * C, 256)), block(256);
    if (is_bf16) sigmoid_gate_kernel<bf16><<<grid, block, 0, st>>>(
        (bf16*)y, (const bf16*)gate, gs, rows, C, vec);
    else sigmoid_gate_kernel<float><<<grid, block, 0, st>>>(
        (float*)y, (const float*)gate, gs, rows, C, vec);
    return (int)hipGetLastError();
}

int nx_scaled_residual(float* x, const void* y0, const float* w0, int n0, const void* y1,
                       const float* w1, int n1, const void* y2, const float* w2, int n2,
                       int is_bf16, float eps, long rows, int C, hipStream_t st) {
    if (rows <= 0) return 0;
    if (!y0 || !w0 || (y1 && !w1) || (y2 && !w2)) return -1;
    dim3 grid((unsigned)rows), block(LN_THREADS);
    const bool al = (C % 8) == 0 && C <= LN_THREADS * 8 * 4 && ((uintptr_t)x % 16) == 0 &&
        ((uintptr_t)y0 % 16) == 0 && ((uintptr_t)y1 % 16) == 0 && ((uintptr_t)y2 % 16) == 0 &&
        ((uintptr_t)w0 % 16) == 0 && ((uintptr_t)w1 % 16) == 0 && ((uintptr_t)w2 % 16) == 0;
    if (al) {
#define SRV(T, NVV) scaled_residual_vec_kernel<T, NVV><<<grid, block, 0, st>>>( \
        x, (const T*)y0, w0, n0, (const T*)y1, w1, n1, (const T*)y2, w2, n2, eps, C)
#define SRN(T) do { if (C <= LN_THREADS * 8) SRV(T, 1); else if (C <= LN_THREADS * 16) SRV(T, 2); \
                    else SRV(T, 4); } while (0)
        if (is_bf16) SRN(bf16); else SRN(float);
#undef SRN
#undef SRV
        return (int)hipGetLastError();
    }
    if (is_bf16) scaled_residual_kernel<bf16><<<grid, block, 0, st>>>(
        x, (const bf16*)y0, w0, n0, (const bf16*)y1, w1, n1, (const bf16*)y2, w2, n2, eps, C);
    else scaled_residual_kernel<float><<<grid, block, 0, st>>>(
        x, (const float*)y0, w0, n0, (const float*)y1, w1, n1, (const float*)y2, w2, n2, eps, C);
    return (int)hipGetLastError();
}

int nx_embed_pos(const void* emb, const void* table, int is_bf16, const int* pos, float* out,
                 long ntok, int C, int rows_in_table, hipStream_t st) {
    if (ntok * C <= 0) return 0;
    if (rows_in_table <= 0) return -1;
    dim3 grid(grid_for(ntok * C, 256)), block(256);
    if (is_bf16) embed_pos_kernel<bf16><<<grid, block, 0, st>>>(
        (const bf16*)emb, (const bf16*)table, pos, out, ntok, C, rows_in_table);
    else embed_pos_kernel<float><<<grid, block, 0, st>>>(
        (const float*)emb, (const float*)table, pos, out, ntok, C, rows_in_table);
    return (int)hipGetLastError();
}

int nx_bigram_embed(const long long* ids, const int* pos, const int* seq, const int* nvalid,
                    const void* emb, const void* table, int is_bf16, int* last, long long mul_prev,
                    long long mul_cur, long long buckets, int vocab, float* out, int B, int S,
                    int C, hipStream_t st) {
    if ((long)B * S * C <= 0) return 0;
    if (buckets <= 0 || vocab <= 0) return -1;
    dim3 grid((unsigned)((long)B * S)), block(256);
    const int vec = (C % 8) == 0 && ((uintptr_t)emb % 16) == 0 && ((uintptr_t)table % 16) == 0 &&
                    ((uintptr_t)out % 16) == 0;
    if (is_bf16) bigram_embed_kernel<bf16><<<grid, block, 0, st>>>(
        ids, pos, seq, nvalid, (const bf16*)emb, (const bf16*)table, last, mul_prev, mul_cur,
        buckets, vocab, out, S, C, vec);
    else bigram_embed_kernel<float><<<grid, block, 0, st>>>(
        ids, pos, seq, nvalid, (const float*)emb, (const float*)table, last, mul_prev, mul_cur,
        buckets, vocab, out, S, C, vec);
    return (int)hipGetLastError();
}

int nx_token_gate(const void* z, long zs, const long long* ids, const void* table, long ts,
                  int off, int vocab, int is_bf16, void* out, long rows, int C, hipStream_t st) {
    if (rows * C <= 0) return 0;
    if (vocab <= 0 || off < 0 || (long)off + C > ts) return -1;
    dim3 grid(grid_for(rows * C, 256)), block(256);
    if (is_bf16) token_gate_kernel<bf16><<<grid, block, 0, st>>>(
        (const bf16*)z, zs, ids, (const bf16*)table, ts, off, vocab, (bf16*)out, rows, C);
    else token_gate_kernel<float><<<grid, block, 0, st>>>(
        (const float*)z, zs, ids, (const float*)table, ts, off, vocab, (float*)out, rows, C);
    return (int)hipGetLastError();
}

int nx_token_gate_proj(const void* x, long xs, const void* wg, int K, const long long* ids,
                       const void* table, long ts, int off, int vocab, void* out, long rows, int C,
                       hipStream_t st) {
    if (rows * C <= 0) return 0;
    if (vocab <= 0 || off < 0 || (long)off + C > ts || K <= 0 || (K % 8) || (xs % 8) ||
        ((uintptr_t)x % 16) || ((uintptr_t)wg % 16) || (rows + 15) / 16 > 65535) return -1;
    dim3 grid((C + 15) / 16, (unsigned)((rows + 15) / 16)), block(512);
    token_gate_proj_kernel<<<grid, block, 0, st>>>((const bf16*)x, xs, (const bf16*)wg, K, ids,
                                                   (const bf16*)table, ts, off, vocab, (bf16*)out,
                                                   rows, C);
    return (int)hipGetLastError();
}

int nx_head_product(const void* a, const void* w, void* out, int T, int H, int K, int N,
                    hipStream_t st) {
    if ((long)T * H * N <= 0) return 0;
    if (K <= 0 || (K % 8) || ((uintptr_t)a % 16) || ((uintptr_t)w % 16) || H > 65535) return -1;
    dim3 grid((N + 15) / 16, H, (T + 63) / 64), block(256);
    head_product_kernel<<<grid, block, 0, st>>>((const bf16*)a, (const bf16*)w, (bf16*)out, T, H,
                                                K, N);
    return (int)hipGetLastError();
}

int nx_hyper_step(const float* xin, long xrow, long xstr, const void* y, int is_bf16,
                  const float* mix, const float* wout, float* xout, const float* win,
                  const float* nw, float eps, void* hout, float* uout, float* scratch, long rows,
                  int NS, int C, hipStream_t st) {
    if (rows <= 0) return 0;
    if (C <= 0 || NS <= 0 || !xin || (y && (!mix || !wout)) || (nw ? !hout : !uout)) return -1;
    dim3 grid((unsigned)rows), block(LN_THREADS);
    const bool vec = (C % 4) == 0 && (xrow % 4) == 0 && (xstr % 4) == 0 && NS <= 4 &&
                     C <= LN_THREADS * 32 &&
                     (((uintptr_t)xin | (uintptr_t)xout | (uintptr_t)y | (uintptr_t)nw |
                       (uintptr_t)hout | (uintptr_t)uout) % 16) == 0;
    if (!vec && ((y && xout == xin) || (nw && !scratch))) return -2;
#define HSV(T, N, V) hyper_step_vec_kernel<T, N, V><<<grid, block, 0, st>>>( \
        xin, xrow, xstr, (const T*)y, mix, wout, xout, win, nw, eps, (T*)hout, uout, C)
#define HSN(T, N) do { if (C <= LN_THREADS * 4) HSV(T, N, 1); else if (C <= LN_THREADS * 8) HSV(T, N, 2); \
        else if (C <= LN_THREADS * 16) HSV(T, N, 4); else HSV(T, N, 8); } while (0)
#define HS(T) do { if (!vec) hyper_step_kernel<T><<<grid, block, 0, st>>>( \
            xin, xrow, xstr, (const T*)y, mix, wout, xout, win, nw, eps, (T*)hout, uout, scratch, \
            NS, C); \
        else if (NS == 1) HSN(T, 1); else if (NS == 2) HSN(T, 2); else if (NS == 3) HSN(T, 3); \
        else HSN(T, 4); } while (0)
    if (is_bf16) HS(bf16); else HS(float);
#undef HS
#undef HSN
#undef HSV
    return (int)hipGetLastError();
}

int nx_qkv_rows(const void* q, long qs, const void* k, long ks, const void* v, long vs,
                const void* vf, long vfs, const float* lam, int is_bf16, const int* pos,
                const int* slots, const float* inv_freq, int half, int unorm, float eps, void* qo,
                void* kc, void* vc, long nslots, long ntok, int H, int G, int D, int Dv,
                hipStream_t st) {
    if (ntok <= 0) return 0;
    if (H <= 0 || G <= 0 || D <= 0 || Dv <= 0 || half < 0 || 2 * half > D || half > HN_MAXC / 2 ||
        (half > 0 && !inv_freq) || (vf && !lam)) return -1;
    const int vecn = is_bf16 ? 8 : 4;
    const bool vec = (D % 8) == 0 && D <= 8 * WAVE && (half % 8) == 0 && ((G * Dv) % 8) == 0 &&
                     (qs % vecn) == 0 && (ks % vecn) == 0 && (vs % vecn) == 0 && (vfs % vecn) == 0 &&
                     (((uintptr_t)q | (uintptr_t)k | (uintptr_t)v | (uintptr_t)vf | (uintptr_t)qo |
                       (uintptr_t)kc | (uintptr_t)vc) % 16) == 0;
    int lanes = 1;
    while (lanes * 8 < D) lanes *= 2;
    dim3 grid((unsigned)ntok), block(256);
#define QK(T) do { if (vec) qkv_rows_vec_kernel<T><<<grid, block, 0, st>>>( \
            (const T*)q, qs, (const T*)k, ks, (const T*)v, vs, (const T*)vf, vfs, lam, pos, slots, \
            inv_freq, half, unorm, eps, (T*)qo, (T*)kc, (T*)vc, nslots, H, G, D, Dv, lanes); \
        else qkv_rows_kernel<T><<<grid, block, 0, st>>>( \
            (const T*)q, qs, (const T*)k, ks, (const T*)v, vs, (const T*)vf, vfs, lam, pos, slots, \
            inv_freq, half, unorm, eps, (T*)qo, (T*)kc, (T*)vc, nslots, H, G, D, Dv); } while (0)
    if (is_bf16) QK(bf16); else QK(float);
#undef QK
    return (int)hipGetLastError();
}

int nx_mlstm_gates(const void* zi, long zis, const void* zf, long zfs, int is_bf16,
                   const float* bi, const float* bf, float cap, float* mstate, const int* pos,
                   const int* seq, const int* nvalid, float* ld, float* wt, float* mx, int B,
                   int S, int H, hipStream_t st) {
    if ((long)B * S <= 0) return 0;
    if (H <= 0 || B > 65535 || !bi || !bf || !(cap > 0.f)) return -1;
    dim3 grid(H, B), block(MG_THREADS);
#define MG(T) mlstm_gates_kernel<T><<<grid, block, 0, st>>>( \
        (const T*)zi, zis, (const T*)zf, zfs, bi, bf, cap, mstate, pos, seq, nvalid, ld, wt, mx, S, H)
    if (is_bf16) MG(bf16); else MG(float);
#undef MG
    return (int)hipGetLastError();
}

int nx_mlstm_readout(const float* o, const float* mx, const void* gate, long gs, int is_bf16,
                     const float* nw, float eps, const int* pos, void* out, long rows, int H,
                     int Dv, hipStream_t st) {
    if (rows <= 0) return 0;
    if (H <= 0 || Dv <= 0 || !nw) return -1;
    dim3 grid((unsigned)((rows * H + 3) / 4)), block(4 * WAVE);
    if (is_bf16) mlstm_readout_kernel<bf16><<<grid, block, 0, st>>>(
        o, mx, (const bf16*)gate, gs, nw, eps, pos, (bf16*)out, rows, H, Dv);
    else mlstm_readout_kernel<float><<<grid, block, 0, st>>>(
        o, mx, (const float*)gate, gs, nw, eps, pos, (float*)out, rows, H, Dv);
    return (int)hipGetLastError();
}

// single-token steps; key channels up to 256
int nx_mlstm_decode(const void* q, long qs, const void* k, long ks, const void* v, long vs,
                    const void* zi, long zis, const void* zf, long zfs, int is_bf16,
                    const float* bi, const float* bf, float cap, float k_scale, const void* gate,
                    long gs, const float* nw, float eps, float* state, float* mstate,
                    const int* pos, const int* seq, void* out, int B, int H, int D, int Dv,
                    hipStream_t st) {
    if (B <= 0) return 0;
    if (H <= 0 || D <= 0 || D > 4 * WAVE || Dv <= 0 || Dv > 8192 || B > 65535 || !bi || !bf ||
        !nw || !(cap > 0.f)) return -1;
    const int vec = (D % 4) == 0 && ((uintptr_t)state % 16) == 0;
    int lanes = 1;
    while (lanes * 4 < D) lanes *= 2;
    dim3 grid(H, B), block(MD_THREADS);
    const size_t sh = (size_t)(Dv + 1) * sizeof(float);
#define MDK(T) mlstm_decode_kernel<T><<<grid, block, sh, st>>>( \
        (const T*)q, qs, (const T*)k, ks, (const T*)v, vs, (const T*)zi, zis, (const T*)zf, zfs, \
        bi, bf, cap, k_scale, (const T*)gate, gs, nw, eps, state, mstate, pos, seq, (T*)out, H, D, \
        Dv, lanes, vec)
    if (is_bf16) MDK(bf16); else MDK(float);
#undef MDK
    return (int)hipGetLastError();
}

// chunked form: bf16 q/k/v/gate/out, D and Dv multiples of 8 up to 128; ws holds
// (B, chunks, H, Dv + 1, D), wdec (B, chunks, H)
int nx_mlstm_chunked(const void* q, long qs, const void* k, long ks, const void* v, long vs,
                     const float* ld, const float* wt, const float* mx, float k_scale,
                     const void* gate, long gs, const float* nw, float eps, float* state,
                     const int* pos, const int* seq, const int* nvalid, float* ws, float* wdec,
                     void* out, int B, int S, int H, int D, int Dv, hipStream_t st) {
    if ((long)B * S <= 0) return 0;
    if (D <= 0 || Dv <= 0 || D > 128 || Dv > 128 || (D % 8) || (Dv % 8)) return -1;
    if ((qs % 8) || (ks % 8) || (vs % 8) || (gs % 8) ||
        (((uintptr_t)q | (uintptr_t)k | (uintptr_t)v | (uintptr_t)gate | (uintptr_t)ws |
          (uintptr_t)out) % 16) || !gate || !nw) return -2;
    const int nc = (S + GC_N - 1) / GC_N;
    if (H > 65535 || B > 65535) return -3;
    dim3 grid(nc, H, B), block(256);
    const long per_head = (long)(Dv + 1) * D;
#define MC(DPV, NT) do { \
        constexpr int DPB = DPV < 64 ? DPV : 64; \
        constexpr size_t qk = 2 * GC_N * (DPV + 8) * 2 > GC_N * (NT * 16 + 4) * 4 \
            ? 2 * GC_N * (DPV + 8) * 2 : GC_N * (NT * 16 + 4) * 4; \
        const size_t lsh = qk + (size_t)(NT * 16 + 2 * GC_N) * GC_VS * 2 + 7 * GC_N * 4; \
        static bool attr_set = false; \
        if (!attr_set) { \
            if (hipFuncSetAttribute((const void*)mlstm_chunk_out_kernel<DPV, NT>, \
                    hipFuncAttributeMaxDynamicSharedMemorySize, (int)lsh) != hipSuccess) return -5; \
            attr_set = true; \
        } \
        dim3 gst(nc * ((D + DPB - 1) / DPB), H, B); \
        mlstm_chunk_state_kernel<DPB, NT><<<gst, block, 0, st>>>( \
            (const bf16*)k, ks, (const bf16*)v, vs, ld, wt, k_scale, seq, nvalid, ws, wdec, S, H, \
            D, Dv, nc); \
        gla_chunk_link_kernel<<<grid_for((long)B * H * per_head, 256), 256, 0, st>>>( \
            ws, wdec, state, pos, seq, nvalid, B, S, H, 1, per_head, nc); \
        mlstm_chunk_out_kernel<DPV, NT><<<grid, block, lsh, st>>>( \
            (const bf16*)q, qs, (const bf16*)k, ks, (const bf16*)v, vs, ld, wt, mx, k_scale, \
            (const bf16*)gate, gs, nw, eps, seq, nvalid, ws, (bf16*)out, S, H, D, Dv, nc); } while (0)
#define MCN(DPV) do { if (Dv <= 64) MC(DPV, 4); else MC(DPV, 8); } while (0)
    if (D <= 32) MCN(32); else if (D <= 64) MCN(64); else MCN(128);
#undef MCN
#undef MC
    return (int)hipGetLastError();
}

}  // extern "C"
