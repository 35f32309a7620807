// hybrid_rows.hip: what attention layers do to whole projection rows between the input GEMM and the attention kernels, in
// one launch (ops/hybrid.py row_rope_append): a short causal convolution over time per query / key channel whose last
// inputs are carried per sequence, or an RMS norm over a token's whole query (key) projection before it is split into
// heads; rotary positions; the queries as a GEMM-side operand and keys and values into the paged pools. Without a value
// projection the values are the keys as they enter the rotation.
//
// A block serves one token and one part: some or all of its query items, of its key items, or its value heads. An ITEM is a
// rotation pair, or one number outside the rotated part: a pair's two numbers stay in one thread and the row needs no LDS.
// With whole-row norms a part is a whole row (up to blockDim.x * RK items wait in registers between the statistics and the
// rotation, longer rows are read again); without them it is blockDim.x * RK items, so that a single token spreads over
// several CUs. All taps' inputs of all items are requested together (a tap before the chunk's first row points into the
// carried inputs, one before the sequence's start into anything and is dropped), and a single new token rolls its
// channels' carried inputs from those same registers. Sine and cosine are computed once per block and pair and shared by
// the heads through LDS. Everything is fp32 up to the stores.
#include "../mx_common.h"

namespace {

template <bool B16>
MX_DEV void st_elem(void* p, long i, float v) {
    if constexpr (B16) ((bf16_t*)p)[i] = f32_to_bf16(v);
    else ((float*)p)[i] = v;
}

struct RowRope {
    const float *q, *k, *v;  // v == nullptr: the values are the keys before the rotation; k == nullptr: queries only
    int ldq, ldk, ldv;
    const int *positions, *slots;
    int H, G, dk, dv, rot, half;
    const float* freqs;  // [rot / 2]
    float mag;
    const float *qw, *kw;  // whole-row norm weights [H * dk], [G * dk] (null: no norm)
    float eps;
    const float* cw;  // convolution weights [taps, C] over C = (H + G) * dk channels, queries first (null: none)
    int taps, C;
    float* tails;  // [slots, taps - 1, C]
    const int* state;
    int n_dec;
    const int* pf_cu;
    int n_pf;
    void* qo;
    int ldqo;
    void *kc, *vc;
};

// TAPS: 1 without a convolution, else the bound of the tap loops (a.taps <= TAPS). grid (T, bq + bk + values)
template <bool Q16, bool C16, int TAPS, int RK>
__global__ __launch_bounds__(1024) void row_rope_append_kernel(RowRope a, int bq, int bk) {
    extern __shared__ float trig[];  // [rot / 2] cosines, [rot / 2] sines
    __shared__ float red[16];
    const int t = blockIdx.x, nt = blockDim.x, tid = threadIdx.x;
    const bool isq = (int)blockIdx.y < bq;
    const long slot = isq ? 0 : a.slots[t];
    if ((int)blockIdx.y >= bq + bk) {
        if (slot < 0) return;
        const float* src = a.v + (long)t * a.ldv;
        const int n = a.G * a.dv;
        for (int c = tid; c < n; c += nt) st_elem<C16>(a.vc, slot * n + c, src[c]);
        return;
    }
    const int part = isq ? blockIdx.y : blockIdx.y - bq, parts = isq ? bq : bk;
    const int heads = isq ? a.H : a.G;
    const int n2 = a.rot >> 1, per = a.dk - n2;  // items per head: n2 pairs, then the unrotated numbers
    const int n_items = heads * per;
    const int ld = isq ? a.ldq : a.ldk;
    const float* src = (isq ? a.q : a.k) + (long)t * ld;
    const float* w = isq ? a.qw : a.kw;
    const int ch0 = isq ? 0 : a.H * a.dk;  // first convolution channel of the part
    const float pos = (float)a.positions[t];
    for (int i = tid; i < n2; i += nt) {
        float s, c;
        sincosf(pos * a.freqs[i], &s, &c);
        trig[i] = c * a.mag;
        trig[n2 + i] = s * a.mag;
    }
    const float* in[TAPS];  // the part's inputs b rows back
    bool live[TAPS];        // false: before the sequence's start
    float* roll = nullptr;  // a single new token's carried inputs
    in[0] = src;
    live[0] = true;
    if constexpr (TAPS > 1) {
        int s, since = 0;  // the row's sequence, rows of its chunk before it
        if (t < a.n_dec) {
            s = t;
        } else {
            int lo = 0, hi = a.n_pf - 1;  // last s with pf_cu[s] <= t - n_dec
            while (lo < hi) {
                const int mid = (lo + hi + 1) >> 1;
                if (a.pf_cu[mid] <= t - a.n_dec) lo = mid;
                else hi = mid - 1;
            }
            s = a.n_dec + lo;
            since = t - a.n_dec - a.pf_cu[lo];
        }
        const int sl = a.state[s];
        float* tail = a.tails + (long)max(sl, 0) * (a.taps - 1) * a.C + ch0;
        const bool carried = sl >= 0 && a.positions[t - since] != 0;
        if (sl >= 0 && t < a.n_dec && a.taps > 1) roll = tail;
#pragma unroll
        for (int b = 1; b < TAPS; ++b) {
            const bool tap = b < a.taps, here = b <= since;
            live[b] = tap && (here || carried);
            in[b] = !live[b] ? src : here ? src - (long)b * ld : tail + (long)(a.taps - 1 - b + since) * a.C;
        }
    }
    auto locate = [&](int it, int& e0, int& e1, int& u) {
        const int hd = it / per;
        u = it - hd * per;
        const bool pair = u < n2;
        e0 = hd * a.dk + (pair ? (a.half ? u : 2 * u) : u + n2);
        e1 = pair ? (a.half ? e0 + n2 : e0 + 1) : e0;
    };
    float x0[RK], x1[RK];
    // the items from `base` on, into x0 / x1; returns the thread's sum of squares
    auto load = [&](int base, bool last) {
        float r0[RK][TAPS], r1[RK][TAPS];
#pragma unroll
        for (int r = 0; r < RK; ++r) {
            int e0, e1, u;
            locate(min(base + tid + r * nt, n_items - 1), e0, e1, u);  // clamped: no branch between the loads
#pragma unroll
            for (int b = 0; b < TAPS; ++b) {
                r0[r][b] = in[b][e0];
                r1[r][b] = in[b][e1];
            }
        }
        if constexpr (TAPS > 1) {
            float ss = 0.f;
#pragma unroll
            for (int r = 0; r < RK; ++r) {
                int e0, e1, u;
                locate(min(base + tid + r * nt, n_items - 1), e0, e1, u);
                x0[r] = x1[r] = 0.f;
#pragma unroll
                for (int b = TAPS - 1; b >= 0; --b) {
                    const float* cw = a.cw + (long)max(a.taps - 1 - b, 0) * a.C + ch0;
                    const float w0 = cw[e0], w1 = cw[e1];
                    x0[r] += w0 * (live[b] ? r0[r][b] : 0.f);
                    x1[r] += w1 * (live[b] ? r1[r][b] : 0.f);
                }
                if (base + tid + r * nt < n_items) ss += x0[r] * x0[r] + (u < n2 ? x1[r] * x1[r] : 0.f);
            }
            if (last && roll) {
#pragma unroll
                for (int r = 0; r < RK; ++r) {
                    const int it = base + tid + r * nt;
                    int e0, e1, u;
                    locate(min(it, n_items - 1), e0, e1, u);
                    if (it < n_items) {
#pragma unroll
                        for (int b = 0; b < TAPS - 1; ++b) {
                            if (b < a.taps - 1) {
                                roll[(long)(a.taps - 2 - b) * a.C + e0] = live[b] ? r0[r][b] : 0.f;
                                if (u < n2) roll[(long)(a.taps - 2 - b) * a.C + e1] = live[b] ? r1[r][b] : 0.f;
                            }
                        }
                    }
                }
            }
            return ss;
        } else {
            float ss = 0.f;
#pragma unroll
            for (int r = 0; r < RK; ++r) {
                const int it = base + tid + r * nt;
                x0[r] = r0[r][0];
                x1[r] = r1[r][0];
                if (it < n_items) ss += x0[r] * x0[r] + (it % per < n2 ? x1[r] * x1[r] : 0.f);
            }
            return ss;
        }
    };
    const int stride = nt * RK;
    const bool cached = w && n_items <= stride;
    float sc = 1.f;
    if (w) {
        float ss = 0.f;
        if (cached) ss = load(0, true);
        else
            for (int base = 0; base < n_items; base += stride) ss += load(base, false);
        ss = wave_sum(ss);
        if ((tid & 63) == 0) red[tid >> 6] = ss;
    } else {
        load(part * stride, true);  // requested before the wait for the angles
    }
    __syncthreads();  // the statistics and the angles
    if (w) {
        float ss = 0.f;
        for (int i = 0; i < nt >> 6; ++i) ss += red[i];
        sc = 1.f / sqrtf(ss / (float)(heads * a.dk) + a.eps);
    }
    const bool tied = !isq && !a.v;
    const long row_q = (long)t * a.ldqo, row_c = slot * (long)(a.G * a.dk);
    for (int base = part * stride; base < n_items; base += parts * stride) {
        if (w ? !cached : base != part * stride) load(base, true);
#pragma unroll
        for (int r = 0; r < RK; ++r) {
            const int it = base + tid + r * nt;
            if (it >= n_items) break;
            int e0, e1, u;
            locate(it, e0, e1, u);
            const bool pair = u < n2;
            float y0 = x0[r] * sc, y1 = x1[r] * sc;
            if (w) {
                y0 *= w[e0];
                y1 *= w[e1];
            }
            float z0 = y0, z1 = y1;
            if (pair) {
                const float c = trig[u], s = trig[n2 + u];
                z0 = y0 * c - y1 * s;
                z1 = y1 * c + y0 * s;
            }
            if (isq) {
                st_elem<Q16>(a.qo, row_q + e0, z0);
                if (pair) st_elem<Q16>(a.qo, row_q + e1, z1);
            } else if (slot >= 0) {
                st_elem<C16>(a.kc, row_c + e0, z0);
                if (pair) st_elem<C16>(a.kc, row_c + e1, z1);
                if (tied) {
                    st_elem<C16>(a.vc, row_c + e0, y0);
                    if (pair) st_elem<C16>(a.vc, row_c + e1, y1);
                }
            }
        }
    }
}

// grid (ceil(C / 256), chunks), launched after the rows: a chunk's newest taps - 1 inputs become the sequence's carried
// ones. Channels 0 .. nq - 1 come from q, the others from k. Single new tokens have rolled theirs.
__global__ __launch_bounds__(256) void row_tails_kernel(RowRope a, int nq) {
    const int c = blockIdx.x * 256 + threadIdx.x, k = blockIdx.y, nt = a.taps - 1;
    const int row0 = a.n_dec + a.pf_cu[k], n = a.pf_cu[k + 1] - a.pf_cu[k], slot = a.state[a.n_dec + k];
    if (c >= a.C || n <= 0 || slot < 0) return;
    const bool fresh = a.positions[row0] == 0;
    const float* src = c < nq ? a.q + c : a.k + (c - nq);
    const int ld = c < nq ? a.ldq : a.ldk;
    float* tail = a.tails + (long)slot * nt * a.C + c;
    for (int i = 0; i < nt; ++i) {
        const int tau = n - nt + i;
        float v = 0.f;
        if (tau >= 0) v = src[(long)(row0 + tau) * ld];
        else if (!fresh) v = tail[(long)(nt + tau) * a.C];  // index n + i > i: not yet overwritten
        tail[(long)i * a.C] = v;
    }
}

}  // namespace

#define MXH_CHECK(cond) \
    if (!(cond)) return (int)hipErrorInvalidValue

extern "C" int mxh_row_rope_append(const float* q, int ldq, const float* k, int ldk, const float* v, int ldv,
                                   const int* positions, const int* slots, int H, int G, int dk, int dv, int rot, int half,
                                   const float* freqs, float mag, const float* qw, const float* kw, float eps,
                                   const float* cw, int taps, float* tails, const int* state, int n_dec, const int* pf_cu,
                                   int n_pf, void* qo, int ldqo, int q16, void* kc, void* vc, int c16, int T,
                                   hipStream_t st) {
    if (T <= 0) return 0;
    MXH_CHECK(q && positions && slots && qo && H > 0 && dk > 0 && dv > 0 && rot >= 0 && rot <= dk && rot % 2 == 0);
    MXH_CHECK((rot == 0 || freqs) && rot <= 8192 && ldq >= H * dk && ldqo >= H * dk && H * (long)dk < (1L << 30));
    MXH_CHECK(k ? (G > 0 && kc && vc && ldk >= G * dk && (v ? ldv >= G * dv : dv == dk)) : !v && !kw);
    MXH_CHECK(!k || !qw == !kw);
    const int g = k ? G : 0;
    MXH_CHECK(!cw || (taps >= 1 && taps <= 16 && tails && state && n_dec >= 0 && n_pf >= 0 && (n_pf == 0 || pf_cu) &&
                      n_dec <= T && (n_pf > 0 || n_dec == T)));
    RowRope a = {q,  k,  v,   ldq, ldk, ldv,  positions, slots, H, g, dk, dv, rot, half, freqs, mag,
                 qw, kw, eps, cw,  cw ? taps : 0, (H + g) * dk, tails, state, n_dec, pf_cu, n_pf, qo, ldqo, kc, vc};
    constexpr int RK = 4;
    const int per = dk - rot / 2, items = max(H, g) * per;
    // whole rows for the norms, else 512 items (two per thread) to a block
    const int nt = qw && items > 1024 ? 1024 : 256;
    const int bq = qw ? 1 : (H * per + 511) / 512, bk = !k ? 0 : kw ? 1 : (g * per + 511) / 512;
    MXH_CHECK(bq + bk < 65535);
    const dim3 grid(T, bq + bk + (v ? 1 : 0));
    const size_t sh = rot * sizeof(float);
#define GO2(Q, C_, TP, R_) row_rope_append_kernel<Q, C_, TP, R_><<<grid, nt, sh, st>>>(a, bq, bk)
#define GO1(Q, C_, TP)             \
    do {                           \
        if (qw) GO2(Q, C_, TP, RK); \
        else GO2(Q, C_, TP, 2);    \
    } while (0)
#define GO(Q, C_)                        \
    do {                                 \
        if (!cw) GO1(Q, C_, 1);          \
        else if (taps <= 4) GO1(Q, C_, 4); \
        else GO2(Q, C_, 16, 2);          \
    } while (0)
    if (q16 && c16) GO(true, true);
    else if (!q16 && !c16) GO(false, false);
    else return (int)hipErrorInvalidValue;
#undef GO
#undef GO1
#undef GO2
    if (cw && taps > 1 && n_pf > 0)
        row_tails_kernel<<<dim3((a.C + 255) / 256, n_pf), 256, 0, st>>>(a, H * dk);
    return (int)hipGetLastError();
}
